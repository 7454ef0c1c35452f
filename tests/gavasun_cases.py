"""Gavasun test bodies, shared by the CPU tests (torch twin of the executor: host logic) and the GPU tests (HIP
kernels). Every case builds its own small configuration with random weights, runs it through the engine
(`StackRunner`, its block pool, slots and step function) and compares with the plain float64 implementation in
`gavasun_oracle.py`."""
from __future__ import annotations

import numpy as np

import gavasun_oracle as oracle
from bizulix_cases import Model as _Model
from bizulix_cases import layer_trail, rel_err, run_cuts, tokens  # noqa: F401  (re-exported for the tests)
from ollama_operator_amd.models.config import (ACT_GELU_UP, ACT_SILU, BLOCK_PRENORM, FF_GLU, FF_MOE, GATE_ELEMENT, MIX_ATTENTION,
                                               MIX_DELTA, MIX_LATENT, QK_NORM_WHOLE_FIRST, ROUTE_SOFTMAX_SCORES, LayerSpec, MixerSpec,
                                               MoESpec, StackConfig)


def yarn(factor=3.0, fast=8.0, slow=1.0, original=64):
    return ("yarn", float(factor), float(fast), float(slow), float(original))


def delta(heads=4, kv_heads=2, dim=8, vdim=14, conv=4):
    return MixerSpec(kind=MIX_DELTA, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv, conv_ring=True, head_decay=True,
                     gate=GATE_ELEMENT)


def latent(heads=3, dim=10, rot_dim=6, vdim=12, kv_rank=20, q_rank=24, scale=0.3, window=13, base=500.0, scaling=yarn(), rot=True):
    return MixerSpec(kind=MIX_LATENT, heads=heads, kv_heads=1, dim=dim, vdim=vdim, scale=scale, rot_dim=rot_dim, kv_rank=kv_rank,
                     q_rank=q_rank, rot_pairs=True, window=window, rot_dims=rot_dim if rot else 0, rot_base=base if rot else 10000.0,
                     rot_scaling=scaling if rot else ())


def attn(heads=6, kv_heads=2, dim=16, vdim=12, scale=0.3, chunk=11, conv=3, rot_dims=8, base=2000.0, scaling=yarn(2.0)):
    return MixerSpec(kind=MIX_ATTENTION, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, bias=True, conv=conv,
                     conv_ring=True, qk_norm=QK_NORM_WHOLE_FIRST, chunk=chunk, rot_dims=rot_dims,
                     rot_base=base if rot_dims else 10000.0, rot_scaling=scaling if rot_dims else ())


def dense(ff=40):
    return MoESpec(kind=FF_GLU, ff=ff, act=ACT_SILU)


def moe(experts=6, top=2, ff=20, shared=28):
    return MoESpec(kind=FF_MOE, route=ROUTE_SOFTMAX_SCORES, experts=experts, top=top, ff=ff, shared_ff=shared, shared_gate=False,
                   expert_act=ACT_GELU_UP)


def config(layers, width=48, vocab=96, loop=(0, 0, 0), eps=1e-5, scale=1.7):
    return StackConfig(arch="gavasun", n_vocab=vocab, n_embd=width, layers=[LayerSpec(mixer=m, mlp=f) for m, f in layers],
                       loop_start=loop[0], loop_stop=loop[1], loop_times=loop[2], loop_mix=False, norm_eps=eps, norm_plus_one=True,
                       block=BLOCK_PRENORM, embed_scale=scale)


def standard():
    """Every mixer twice with sizes that differ from one another, layers with and without a feed-forward, a looped span over
    a stateful layer and a latent one."""
    return config([(attn(), moe()),
                   (delta(), moe(experts=5, top=3, ff=16, shared=0)),
                   (latent(), dense()),
                   (latent(heads=2, dim=8, rot_dim=4, vdim=20, kv_rank=12, q_rank=8, window=40, base=100.0, scaling=()), None),
                   (delta(heads=3, kv_heads=1, dim=18, vdim=6, conv=2), dense(ff=24)),
                   (attn(heads=4, kv_heads=4, dim=8, vdim=20, chunk=24, conv=2, rot_dims=4, scaling=()), moe(experts=4, top=1))],
                  loop=(1, 3, 2))


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
    def scaling():
        return rng.choice([(), yarn(rng.choice([1.5, 4.0, 16.0]), rng.choice([8.0, 32.0]), 1.0, rng.choice([128, 2048]))])

    def mk_delta():
        G = rng.choice([1, 2, 3])
        return delta(heads=G * rng.choice([1, 2, 3]), kv_heads=G, dim=rng.choice([24, 32, 64, 128]), vdim=rng.choice([32, 48, 128]),
                     conv=rng.choice([1, 2, 4, 5]))

    def mk_latent():
        return latent(heads=rng.choice([1, 3, 6]), dim=rng.choice([32, 48, 64]), rot_dim=rng.choice([8, 16, 32]),
                      vdim=rng.choice([32, 80]), kv_rank=rng.choice([64, 96, 112]), q_rank=rng.choice([64, 100]),
                      scale=rng.choice([0.08, 0.15]), window=rng.choice([1, 33, 64, 200, 1000]),
                      base=rng.choice([1e3, 5e4]), scaling=scaling())

    def mk_attn():
        G = rng.choice([1, 2, 4])
        return attn(heads=G * rng.choice([1, 2, 3]), kv_heads=G, dim=rng.choice([32, 64, 72, 128]), vdim=rng.choice([32, 64, 128]),
                    scale=rng.choice([0.08, 0.15]), chunk=rng.choice([1, 33, 64, 200, 1000]), conv=rng.choice([1, 2, 3, 6]),
                    rot_dims=rng.choice([16, 32]), base=rng.choice([1e3, 1e6]), scaling=scaling())

    def mk_ff():
        if rng.random() < 0.4:
            return rng.choice([None, dense(ff=rng.choice([100, 192]))])
        n = rng.choice([4, 9, 16])
        return moe(experts=n, top=rng.randint(1, min(4, n)), ff=rng.choice([64, 96, 100]), shared=rng.choice([0, 64, 100]))

    layers = [(mk(), mk_ff()) for mk in rng.sample([mk_delta, mk_latent, mk_attn, mk_delta, mk_attn], rng.randint(3, 5))]
    a = rng.randint(0, len(layers) - 1)
    return config(layers, width=rng.choice([128, 160, 224, 288]), vocab=rng.choice([500, 777]), eps=rng.choice([1e-5, 1e-6]),
                  loop=rng.choice([(0, 0, 0), (a, rng.randint(a + 1, len(layers)), rng.randint(1, 3))]), scale=rng.choice([1.0, 4.0]))


class Model(_Model):
    def oracle(self, toks):
        z, trail = oracle.forward(self.json, self.tensors, toks)
        return z.numpy(), trail.numpy()
