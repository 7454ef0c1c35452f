"""Rogisun test bodies, shared by the CPU tests (torch twin of the executor: host logic) and the GPU tests (HIP
kernels). Every case builds its own small configuration with random weights, runs it through the engine
(`StackRunner`, its block pool, slots and step function) and compares with the plain float64 implementation in
`rogisun_oracle.py`."""
from __future__ import annotations

import numpy as np

import rogisun_oracle as oracle
from bizulix_cases import Model as _Model
from bizulix_cases import layer_trail, rel_err, run_cuts, tokens  # noqa: F401  (re-exported for the tests)
from ollama_operator_amd.models.config import (ACT_CLAMPED_GLU, BLOCK_PRENORM, FF_MOE, GATE_ELEMENT, GATE_HEAD, MIX_ATTENTION,
                                               MIX_DELTA, MIX_LINEAR, MIX_MAMBA2, ROUTE_SIGMOID_GROUPS, LayerSpec, MixerSpec, MoESpec,
                                               StackConfig)


def linear(decay=(0.6, 0.97, 1.0), dim=12, vdim=10):
    return MixerSpec(kind=MIX_LINEAR, heads=len(decay), kv_heads=len(decay), dim=dim, vdim=vdim, decay=tuple(decay), gate=GATE_ELEMENT)


def mamba(heads=4, vdim=6, state=8, groups=2, conv=3, norm_groups=2):
    return MixerSpec(kind=MIX_MAMBA2, heads=heads, kv_heads=groups, dim=state, vdim=vdim, state=state, groups=groups, conv=conv,
                     norm_groups=norm_groups)


def delta(heads=4, kv_heads=2, dim=8, vdim=14, conv=4, decay_rank=0, gate_rank=0):
    return MixerSpec(kind=MIX_DELTA, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv, decay_rank=decay_rank,
                     gate_rank=gate_rank)


def pair(heads=6, kv_heads=2, dim=16, vdim=12, scale=0.3, chunk=11, left=0.7, right=1.3, r=None):
    return MixerSpec(kind=MIX_ATTENTION, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, chunk=chunk, alibi=True,
                     v_unit=True, gate=GATE_HEAD, left_scale=left, right_scale=right, right=r or delta())


def moe(experts=6, top=2, ff=20, limit=1.2):
    return MoESpec(kind=FF_MOE, route=ROUTE_SIGMOID_GROUPS, experts=experts, top=top, ff=ff, shared_gate=False, route_norm=False,
                   expert_act=ACT_CLAMPED_GLU, limit=limit, scale_input=True)


def config(layers, width=48, vocab=96, eps=1e-5, taps=4):
    return StackConfig(arch="rogisun", n_vocab=vocab, n_embd=width, layers=[LayerSpec(mixer=m, mlp=f) for m, f in layers],
                       norm_eps=eps, block=BLOCK_PRENORM, canon_taps=taps, canon_both=True, tied_head=True)


def standard():
    """Every mixer with sizes that differ from one another, layers with and without a feed-forward, several experts per
    token, the pair layer first and in the middle."""
    return config([(pair(), moe()),
                   (linear(), moe(experts=5, top=3, ff=16, limit=2.5)),
                   (mamba(), None),
                   (pair(heads=4, kv_heads=4, dim=8, vdim=20, chunk=24, left=1.0, right=0.6,
                         r=delta(heads=3, kv_heads=1, dim=18, vdim=6, conv=2)),
                    moe(experts=4, top=1)),
                   (mamba(heads=3, vdim=10, state=12, groups=1, conv=4, norm_groups=3), moe()),
                   (linear(decay=(0.9, 0.3), dim=6, vdim=20), None)])


def check(got, want, dtype, what=""):
    """float32: every row within 1e-4 of the logits' spread. bfloat16 is loose on purpose: a router's close call that
    falls the other way swaps a whole expert, so by the typical row: the median within 6e-2, at most one row in ten (or
    three) over 0.5. The sharp comparisons are the float32 ones."""
    e = rel_err(got, want)
    assert np.isfinite(np.asarray(got)).all(), f"{what}: non-finite logits"
    worst = f"{what}: worst row {int(e.argmax())} off by {e.max():.3g} (median {np.median(e):.3g})"
    if dtype == "float32":
        assert e.max() < 1e-4, worst
    else:
        assert np.median(e) < 6e-2 and (e > 0.5).sum() <= max(3, len(e) // 10), worst


def random_config(rng):
    """A configuration drawn at the scale of a small real model (rng: random.Random)."""
    def mk_linear():
        n = rng.choice([2, 3, 6])
        return linear(decay=[1.0 - 2.0 ** -rng.uniform(0.5, 8) for _ in range(n)], dim=rng.choice([24, 32, 64, 96]),
                      vdim=rng.choice([32, 48, 80]))

    def mk_mamba():
        G = rng.choice([1, 2, 3])
        H = G * rng.choice([1, 2, 4])
        return mamba(heads=H, vdim=rng.choice([16, 32, 48]), state=rng.choice([16, 32, 64, 96]), groups=G, conv=rng.choice([1, 2, 4, 5]),
                     norm_groups=rng.choice([1, G, H]))

    def mk_pair():
        G, Gr = rng.choice([1, 2, 4]), rng.choice([1, 2, 3])
        return pair(heads=G * rng.choice([1, 2, 3]), kv_heads=G, dim=rng.choice([32, 64, 72]), vdim=rng.choice([32, 64]),
                    scale=rng.choice([0.08, 0.15]), chunk=rng.choice([1, 33, 64, 200, 1000]), left=rng.uniform(0.4, 1.5),
                    right=rng.uniform(0.4, 1.5),
                    r=delta(heads=Gr * rng.choice([1, 2]), kv_heads=Gr, dim=rng.choice([24, 32, 64, 128]), vdim=rng.choice([32, 48, 128]),
                            conv=rng.choice([1, 2, 4]), decay_rank=rng.choice([8, 12, 40]), gate_rank=rng.choice([8, 20])))

    def mk_ff():
        n = rng.choice([4, 9, 16])
        return None if rng.random() < 0.2 else moe(experts=n, top=rng.randint(1, min(4, n)), ff=rng.choice([64, 96, 100]),
                                                   limit=rng.choice([0.8, 2.0, 7.0]))

    layers = [(mk(), mk_ff()) for mk in rng.sample([mk_linear, mk_mamba, mk_pair, mk_pair, mk_mamba], rng.randint(3, 5))]
    return config(layers, width=rng.choice([128, 160, 224, 288]), vocab=rng.choice([500, 777]), eps=rng.choice([1e-5, 1e-6]),
                  taps=rng.choice([1, 2, 3, 5]))


class Model(_Model):
    def oracle(self, toks):
        z, trail = oracle.forward(self.json, self.tensors, toks)
        return z.numpy(), trail.numpy()
