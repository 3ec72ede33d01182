"""Sodudra through the ragged stack engine against the plain float64 oracle (oracle/sodudra_oracle.py), on small configurations and
random weights made here.  fp32 engine: tight bound (what summation order can explain), routers with random weights (their decisions
are checked on the oracle not to be close calls at that bound); bfloat16 engine: loose bound, routers rigged so that no decision is
close, and crafted weights where random ones would hide a fault (one far key among hundreds, a sink, a head's gate, a pass's step, a
layer's part of the side embedding)."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import sodudra_oracle as O
from sodudra_cases import as_model, as_tensors, decisive_router, layer, make_config, moe, random_weights, routing_margin
from tolenex_cases import as_f64, bf16_round, rel_err, replay

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32_TOL, BF16_TOL = 3e-5, 5e-2


def has_choice(cfg):
    return any(l.get('mlp') and l['mlp']['router']['top'] < l['mlp']['router']['experts'] for l in cfg['layers'])


def weights_for(cfg, seed, dtype, toks=None):
    """Random weights; for the bfloat16 engine the routers are rigged.  With `toks`, the routers' decisions on them are checked on
    the oracle to stand clear of what the engine's rounding can move; a model with a close call is passed over for the next seed."""
    need = 0.15 if dtype == 'bfloat16' else 2e-5
    for attempt in range(20):
        w = random_weights(cfg, seed + 1000 * attempt)
        if not has_choice(cfg):
            return w
        if dtype == 'bfloat16':
            w = decisive_router(cfg, w, seed)
        if toks is None or all(routing_margin(cfg, w, t) > need for t in (toks.values() if isinstance(toks, dict) else [toks])):
            return w
    raise AssertionError('twenty models in a row with a router decision that is a close call')


def session_for(cfg, w, dtype='float32', max_tokens=1024, max_sequences=4, **kw):
    from tensorrt_llm.runtime import RaggedGenerationSession
    return RaggedGenerationSession(as_model(cfg, w), dtype=dtype, max_tokens=max_tokens, max_sequences=max_sequences, **kw)


def tokens_for(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg['vocab'], n).tolist()


def check(got, want, tol, what=''):
    e = rel_err(got, want)
    assert np.isfinite(got).all(), what
    assert e.max() < tol, f'{what}: worst row {int(e.argmax())} of {len(e)} has relative error {e.max():.3g} (bound {tol})'


def tol_of(dtype):
    return F32_TOL if dtype == 'float32' else BF16_TOL


def to_bf16(x):
    return bf16_round(np.asarray(x, np.float32)).astype(np.float64)


def check_rows(got, toks, w, cfg, dtype, what=''):
    """Every position of a request against the oracle.  fp32: the flat bound.  bfloat16: rows differ in how much rounding moves them -
    where a token input's gate is shut in all its channels, the norm behind it magnifies what rounding left - so a row is held to 3 x
    the most that rounding the oracle's own activations to bfloat16 does to it, to nearest and with two random ditherings (never less
    than the median row's); no row may pass 1.5 x that, and at most one row in fifty (or one) may pass it at all."""
    wf = as_f64(w)
    want = O.logits(toks, wf, cfg)
    if dtype == 'float32':
        return check(got, want, F32_TOL, what)
    moved = np.zeros(len(toks))
    for seed in range(3):
        rng = np.random.default_rng(seed)
        fn = to_bf16 if seed == 0 else lambda x: to_bf16(x * (1.0 + rng.uniform(-2.0 ** -9, 2.0 ** -9, np.shape(x))))
        with O.rounding(fn):
            moved = np.maximum(moved, rel_err(O.logits(toks, wf, cfg), want))
    limit = 3.0 * np.maximum(moved, np.median(moved))
    e = rel_err(got, want)
    assert np.isfinite(got).all(), what
    worst = int((e / limit).argmax())
    assert (e < 1.5 * limit).all(), f'{what}: row {worst} of {len(e)} has relative error {e[worst]:.3g}, its limit is {limit[worst]:.3g}'
    assert (e > limit).sum() <= max(1, len(e) // 50), f'{what}: {(e > limit).sum()} of {len(e)} rows are over their limits'
    assert np.median(e) < 3e-2, f'{what}: the median row is off by {np.median(e):.3g}'


GENERAL = make_config([layer(mlp=moe()), layer(heads=1, dim=8, vdim=16, kv_rank=24, mlp=None), layer(heads=5, dim=10, vdim=6, kv_rank=33, mlp=moe(experts=7, top=3, ff=10, shared=0)),
                       layer(heads=2, vdim=8, mlp=moe(experts=3, top=1, ff=40, shared=9))], loop=(1, 3, 2), eps=3e-6)
# shapes the MFMA tile kernels and the LDS-staged products take in bfloat16; fp32 runs them on the general kernels
TILED = make_config([layer(heads=9, dim=32, vdim=16, kv_rank=128, mlp=moe(experts=8, top=3, ff=64, shared=128)),
                     layer(heads=2, dim=64, vdim=96, kv_rank=256, mlp=moe(experts=4, top=2, ff=128, shared=64)),
                     layer(heads=16, dim=16, vdim=8, kv_rank=64, mlp=moe(experts=16, top=4, ff=64, shared=64))], width=192, vocab=320, loop=(0, 2, 2), side=64)
STACKS = {'general': GENERAL, 'tiled': TILED}

MECHANISMS = {
    'attention_alone': make_config([layer()], side=0),
    'attention_one_head': make_config([layer(heads=1, dim=8, vdim=5, kv_rank=7)], side=0),
    'attention_values_wider_than_keys': make_config([layer(heads=4, dim=4, vdim=40, kv_rank=20)], side=0),
    'attention_many_heads_odd_sizes': make_config([layer(heads=7, dim=6, vdim=10, kv_rank=18)], width=72, side=0),
    'attention_latent_wider_than_the_width': make_config([layer(heads=2, kv_rank=150)], side=0),
    'attention_latent_beyond_512': make_config([layer(heads=2, kv_rank=530)], side=0),
    'attention_large_scale': make_config([layer(scale=1.0)], side=0),
    'moe_alone': make_config([layer(heads=1, dim=4, vdim=4, kv_rank=8, mlp=moe())], side=0),
    'moe_no_shared': make_config([layer(mlp=moe(shared=0))]),
    'moe_top_one': make_config([layer(mlp=moe(experts=5, top=1))]),
    'moe_one_expert': make_config([layer(mlp=moe(experts=1, top=1))]),
    'moe_every_expert': make_config([layer(mlp=moe(experts=4, top=4))]),
    'moe_many_experts': make_config([layer(mlp=moe(experts=70, top=5, ff=9, shared=8))], width=160),
    'moe_thirty_chosen': make_config([layer(mlp=moe(experts=40, top=30, ff=8, shared=16))], width=128),
    'moe_sixteen_chosen': make_config([layer(mlp=moe(experts=20, top=16, ff=8, shared=16))], width=128),
    'moe_equal_shared_and_expert_size': make_config([layer(mlp=moe(ff=32, shared=32))]),
    'moe_tile_sizes': make_config([layer(heads=2, dim=32, vdim=32, kv_rank=32, mlp=moe(experts=4, top=2, ff=128, shared=192))], width=128),
    'side_alone': make_config([layer(heads=1, dim=4, vdim=4, kv_rank=8)]),
    'side_of_one_channel': make_config([layer(), layer()], side=1),
    'side_tile_sizes': make_config([layer(), layer(mlp=moe())], width=128, side=128),
    'no_side': make_config([layer(mlp=moe()), layer()], side=0, loop=(0, 1, 2)),
    'loop_of_everything': make_config([layer(mlp=moe()), layer(heads=2)], loop=(0, 2, 3)),
    'loop_of_the_last_layer': make_config([layer(), layer(mlp=moe())], loop=(1, 2, 2)),
    'loop_of_one_pass': make_config([layer(), layer(mlp=moe()), layer()], loop=(1, 2, 1)),
    'no_loop': make_config([layer(mlp=moe()), layer()]),
    'no_cap': make_config([layer(mlp=moe())], softcap=None, logit_scale=1.7),
    'no_scale': make_config([layer(mlp=moe())], softcap=4.0, logit_scale=1.0),
    'general_stack': GENERAL,
    'tiled_stack': TILED,
    'width_that_is_no_multiple_of_four': make_config([layer(heads=3, dim=7, vdim=5, kv_rank=13, mlp=moe(experts=5, top=2, ff=10, shared=7)),
                                                      layer(heads=2, dim=9, vdim=11, kv_rank=6)], width=70, vocab=131, side=5, loop=(0, 1, 2)),
}
for _r in (32, 64, 96, 128, 192, 256):
    MECHANISMS[f'attention_tile_{_r}'] = make_config([layer(heads=2 if _r % 3 else 8, dim=16, vdim=16, kv_rank=_r)], width=128, side=0)


@pytest.mark.parametrize('name', sorted(MECHANISMS))
@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_each_mechanism_whole_prompt(name, dtype):
    cfg = MECHANISMS[name]
    toks = tokens_for(cfg, 150, 1)  # crosses page borders
    w = weights_for(cfg, len(name), dtype, toks)
    s = session_for(cfg, w, dtype)
    got = replay(s, {'a': toks}, [[('a', len(toks))]])['a']
    check_rows(got, toks, w, cfg, dtype, name)


@pytest.mark.parametrize('name', sorted(MECHANISMS))
@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_each_mechanism_decoded(name, dtype):
    cfg = MECHANISMS[name]
    toks = tokens_for(cfg, 75, 2)
    w = weights_for(cfg, len(name) + 1, dtype, toks)
    s = session_for(cfg, w, dtype)
    got = replay(s, {'a': toks}, [[('a', 60)], [('a', 2)]] + [[('a', 1)]] * 13)['a']
    check_rows(got, toks, w, cfg, dtype, name)


@pytest.mark.parametrize('stack', sorted(STACKS))
@pytest.mark.parametrize('dtype,bound', [('float32', 1e-5), ('bfloat16', 5e-2)])
def test_residual_stream_behind_every_layer_run(stack, dtype, bound):
    """Also that a tap holds the stream before the next pass's step is added."""
    cfg = STACKS[stack]
    toks = tokens_for(cfg, 19, 2)
    w = weights_for(cfg, 3, dtype, toks)
    _, taps = O.forward(toks, as_f64(w), cfg, return_layers=True)
    s = session_for(cfg, w, dtype, debug_mode=True)
    s.step([('a', toks, [0])])
    assert s.engine.layer_runs == len(taps) == len(O.execution(cfg)) > len(cfg['layers'])
    for j, x in enumerate(taps):
        assert np.abs(s.engine.tap(j) - x).max() < bound * np.abs(x).max(), f'layer run {j}'


@pytest.mark.parametrize('stack', sorted(STACKS))
@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_prefill_then_token_by_token(dtype, stack):
    cfg = STACKS[stack]
    toks = tokens_for(cfg, 170, 3)
    w = weights_for(cfg, 5, dtype, toks)
    s = session_for(cfg, w, dtype)
    got = replay(s, {'a': toks}, [[('a', 100)]] + [[('a', 1)]] * 70)['a']
    check_rows(got, toks, w, cfg, dtype)


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
@pytest.mark.parametrize('sizes', [[2] * 40, [3, 61, 2, 64, 1, 5, 2, 58, 1, 1, 2], [63, 2, 63, 1, 1, 66], [1] * 9 + [120, 2], [8, 9, 31, 32, 33, 7, 40]])
@pytest.mark.parametrize('stack', sorted(STACKS))
def test_portions_of_a_prompt(sizes, dtype, stack):
    cfg = STACKS[stack]
    toks = tokens_for(cfg, sum(sizes), 4)
    w = weights_for(cfg, 8, dtype, toks)
    s = session_for(cfg, w, dtype)
    got = replay(s, {'a': toks}, [[('a', n)] for n in sizes])['a']
    check_rows(got, toks, w, cfg, dtype)


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
@pytest.mark.parametrize('stack', sorted(STACKS))
def test_unequal_requests_in_one_batch_equal_each_alone(dtype, stack):
    cfg = STACKS[stack]
    reqs = {'a': tokens_for(cfg, 131, 5), 'b': tokens_for(cfg, 9, 6), 'c': tokens_for(cfg, 66, 7), 'd': tokens_for(cfg, 2, 8)}
    w = weights_for(cfg, 9, dtype, reqs)
    schedule = [[('a', 60), ('b', 2)], [('b', 1), ('a', 5), ('c', 64)], [('c', 1), ('b', 1), ('a', 1), ('d', 2)],
                [('a', 63), ('b', 5), ('c', 1)], [('a', 1)], [('a', 1)]]
    s = session_for(cfg, w, dtype)
    got = replay(s, reqs, schedule)
    for rid, toks in reqs.items():
        check_rows(got[rid], toks, w, cfg, dtype, rid)
    assert not s.live() and s.cache.blocks_manager.num_free_blocks() == s.num_blocks and s.slots.num_free_slots() == 4


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_requests_of_very_unequal_length_decode_side_by_side(dtype):
    """Contexts from 1 to 700 tokens in one decoding step: the key split over workgroups leaves empty shares to the short ones."""
    cfg = TILED
    reqs = {'long': tokens_for(cfg, 718, 90), 'mid': tokens_for(cfg, 75, 91), 'new': tokens_for(cfg, 12, 92)}
    w = weights_for(cfg, 21, dtype, reqs)
    schedule = [[('long', 698)], [('mid', 65), ('long', 1)]] + [[('long', 1), ('mid', 1), ('new', 1)]] * 10 + [[('long', 9), ('new', 2)]]
    s = session_for(cfg, w, dtype, max_tokens=1024)
    got = replay(s, reqs, schedule)
    for rid, toks in reqs.items():
        check_rows(got[rid], toks, w, cfg, dtype, rid)


@pytest.mark.parametrize('wide', ['0', '1'])
def test_both_prompt_forms_of_long_latents(wide, monkeypatch):
    monkeypatch.setenv('TLLM_STACK_WIDE_PREFILL', wide)
    cfg = make_config([layer(heads=3, kv_rank=192), layer(heads=2, kv_rank=256, mlp=moe())], width=128, side=16)
    reqs = {'a': tokens_for(cfg, 300, 95), 'b': tokens_for(cfg, 171, 96)}
    w = weights_for(cfg, 25, 'bfloat16', reqs)
    schedule = [[('a', 129), ('b', 33)], [('a', 1), ('b', 130)], [('a', 150), ('b', 1)], [('a', 20), ('b', 7)]]
    s = session_for(cfg, w, 'bfloat16')
    got = replay(s, reqs, schedule)
    for rid, toks in reqs.items():
        check_rows(got[rid], toks, w, cfg, 'bfloat16', rid)


def test_pages_and_slots_that_are_used_again():
    """A pool of 4 pages and 2 slots serves six requests one after another and side by side: every page is written by several
    requests, and what an earlier one left there must never be seen by a later one."""
    cfg = GENERAL
    s = None
    used_blocks, used_slots = [], []
    w = None
    for rnd in range(3):
        reqs = {f'x{rnd}': tokens_for(cfg, 100 + rnd, 20 + rnd), f'y{rnd}': tokens_for(cfg, 70 - rnd, 30 + rnd)}
        if s is None:
            every = {f'{n}{r}': tokens_for(cfg, *a) for r in range(3) for n, a in (('x', (100 + r, 20 + r)), ('y', (70 - r, 30 + r)))}
            w = weights_for(cfg, 11, 'float32', every)
            s = session_for(cfg, w, 'float32', max_tokens=256, max_sequences=2)
            assert s.num_blocks == 4
        x, y = f'x{rnd}', f'y{rnd}'
        schedule = [[(x, 50), (y, 3)], [(y, len(reqs[y]) - 3), (x, 1)], [(x, len(reqs[x]) - 51)]]
        got = replay(s, reqs, schedule, end_when_done=False)
        for rid in reqs:
            seq = s._seq[rid]
            used_blocks.append(tuple(s.cache.blocks_manager.block_ids(seq)[0]))
            used_slots.append(s.slots.slot_of(seq))
            check(got[rid], O.logits(reqs[rid], as_f64(w), cfg), F32_TOL, rid)
            s.release(rid)
    assert len(set(used_slots)) == 2 and len(used_slots) == 6
    assert len({b for blocks in used_blocks for b in blocks}) == 4 and sum(len(b) for b in used_blocks) == 12


def rigged_latent(n, p_far, seed, C, heads=2, D=16, E=24):
    """One layer whose head 0 is rigged so that the LAST token's query meets the key of the token at p_far with a score far above all
    others, so that dropping, shifting or corrupting it moves the logits at the last position by much more than bfloat16 rounding:
    channel 0 of the residual belongs to the far token and is what channel 0 of the latent reads, channel 1 to the last token, and
    dimension D - 1 of head 0's query reads nothing else, that of its key only channel 0 of the latent."""
    cfg = make_config([layer(heads=heads, dim=D, vdim=E, kv_rank=C)], side=0)
    w = random_weights(cfg, seed)
    rng = np.random.default_rng(seed)
    far_tok = 3
    last_tok = far_tok if p_far == n - 1 else 4
    toks = [int(t) for t in rng.integers(5, cfg['vocab'], n)]
    toks[p_far], toks[-1] = far_tok, last_tok
    w['embed'][:, :2] = 0.0
    w['embed'][far_tok, 0] = w['embed'][last_tok, 1] = 20.0
    w['embed.norm'][:2] = w['l0.norm1'][:2] = 1.0
    w['l0.mix.dkv'][0] = 0.0
    w['l0.mix.dkv'][0, 0] = 4.0
    w['l0.mix.dkv.norm'][0] = 1.0
    w['l0.mix.uk'][D - 1] = 0.0
    w['l0.mix.uk'][D - 1, 0] = 1.0
    w['l0.mix.q'][D - 1] = 0.0
    w['l0.mix.q'][D - 1, 1] = bf16_round(np.float32(0.8 / cfg['layers'][0]['mixer']['scale']))
    w['l0.mix.g'][0] = 0.0
    w['l0.mix.sink'][0] = 2.0
    w['l0.mix.uv'][:E] *= 4.0
    return cfg, w, toks


@pytest.mark.parametrize('p_far', [0, 1, 31, 32, 63, 64, 127, 128, 200, 331])
@pytest.mark.parametrize('dtype,C,heads', [('float32', 40, 2), ('bfloat16', 40, 2), ('bfloat16', 64, 2), ('bfloat16', 256, 9)])
def test_a_far_key_that_decides_the_answer(p_far, dtype, C, heads):
    """In a whole prompt, in a portion that starts behind the far token, decoded alone, and decoded beside another request."""
    cfg, w, toks = rigged_latent(333, p_far, seed=40 + p_far, C=C, heads=heads)
    n, wf = len(toks), as_f64(w)
    want = O.logits(toks, wf, cfg)
    other = list(toks)
    other[p_far] = 7
    moved = rel_err(O.logits(other, wf, cfg)[-1:], want[-1:])[0]
    assert moved > 0.1, f'the rig does not bite: replacing the far token moves the last row by {moved:.3g} only'
    s = session_for(cfg, w, dtype)
    cut = max(p_far + 1, 2)
    check(replay(s, {'w': toks}, [[('w', n)]])['w'][-1:], want[-1:], tol_of(dtype), 'whole')
    check(replay(s, {'p': toks}, [[('p', cut)], [('p', n - cut)]])['p'][-1:], want[-1:], tol_of(dtype), 'portion')
    check(replay(s, {'d': toks}, [[('d', n - 1)], [('d', 1)]])['d'][-1:], want[-1:], tol_of(dtype), 'decoded')
    side = tokens_for(cfg, 4, 77)
    got = replay(s, {'d': toks, 'e': side}, [[('e', 3), ('d', 50)], [('d', n - 51)], [('e', 1), ('d', 1)]])
    check(got['d'][-1:], want[-1:], tol_of(dtype), 'decoded in a batch')


@pytest.mark.parametrize('heads,C', [(3, 40), (9, 128), (33, 256)])
@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_the_sinks_take_their_shares(dtype, heads, C):
    """Sinks as large as the scores and different per head: leaving them out, or handing a head its neighbour's, changes the oracle's
    logits by much; whole prompt, then decoding (where 16 heads are the rows of a tile)."""
    cfg = make_config([layer(heads=heads, dim=16, vdim=8, kv_rank=C)], side=0)
    w = random_weights(cfg, 33)
    w['l0.mix.sink'][:] = bf16_round(np.linspace(1.0, 9.0, heads).astype(np.float32))
    toks = tokens_for(cfg, 70, 34)
    wf = as_f64(w)
    want = O.logits(toks, wf, cfg)
    for wrong in (np.full(heads, -1e9), np.roll(wf['l0.mix.sink'], heads // 2)):
        assert np.median(rel_err(O.logits(toks, dict(wf, **{'l0.mix.sink': wrong}), cfg), want)) > 0.1
    s = session_for(cfg, w, dtype)
    check_rows(replay(s, {'a': toks}, [[('a', 40)]] + [[('a', 1)]] * 30)['a'], toks, w, cfg, dtype)


@pytest.mark.parametrize('heads,C', [(3, 40), (9, 128), (33, 256)])
@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_every_head_has_its_own_gate(dtype, heads, C):
    """Gates nearly open for some heads and nearly shut for others, by token."""
    cfg = make_config([layer(heads=heads, dim=16, vdim=8, kv_rank=C)], side=0)
    w = random_weights(cfg, 35)
    w['l0.mix.g'] *= 4.0
    toks = tokens_for(cfg, 70, 36)
    wf = as_f64(w)
    assert np.median(rel_err(O.logits(toks, dict(wf, **{'l0.mix.g': np.roll(wf['l0.mix.g'], 1, axis=0)}), cfg), O.logits(toks, wf, cfg))) > 0.1
    s = session_for(cfg, w, dtype)
    check_rows(replay(s, {'a': toks}, [[('a', 40)]] + [[('a', 1)]] * 30)['a'], toks, w, cfg, dtype)


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_passes_and_layers_do_not_share_what_is_their_own(dtype):
    """Large, different steps per pass and side parts per layer: swapping two of either moves the oracle's logits by much."""
    cfg = make_config([layer(), layer(heads=2)], loop=(0, 2, 2), side=8)
    w = random_weights(cfg, 37)
    for k in ('loop.step', 'l0.side.norm', 'l1.side.norm'):
        w[k] = w[k] * 4.0
    toks = tokens_for(cfg, 40, 38)
    wf = as_f64(w)
    want = O.logits(toks, wf, cfg)
    assert np.median(rel_err(O.logits(toks, dict(wf, **{'loop.step': wf['loop.step'][::-1]}), cfg), want)) > 0.1
    assert np.median(rel_err(O.logits(toks, dict(wf, **{'side.embed': np.roll(wf['side.embed'], 8, axis=1)}), cfg), want)) > 0.1
    s = session_for(cfg, w, dtype)
    check_rows(replay(s, {'a': toks}, [[('a', 30)]] + [[('a', 1)]] * 10)['a'], toks, w, cfg, dtype)


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_logits_deep_in_the_cap(dtype):
    cfg = make_config([layer(mlp=moe(experts=2, top=2))], softcap=2.0, logit_scale=3.0)
    w = random_weights(cfg, 39)
    toks = tokens_for(cfg, 50, 40)
    s = session_for(cfg, w, dtype)
    got = replay(s, {'a': toks}, [[('a', 45)]] + [[('a', 1)]] * 5)['a']
    assert np.abs(got).max() <= 2.0 and np.abs(got).max() > 1.99
    check_rows(got, toks, w, cfg, dtype)


@pytest.mark.parametrize('stack', sorted(STACKS))
def test_first_tokens_of_a_sequence(stack):
    cfg = STACKS[stack]
    lists = {n: tokens_for(cfg, n, 50 + n) for n in (1, 2, 3, 4, 5)}
    for dtype in ('float32', 'bfloat16'):
        w = weights_for(cfg, 13, dtype, lists)
        s = session_for(cfg, w, dtype)
        for n, toks in lists.items():
            want = O.logits(toks, as_f64(w), cfg)
            check(replay(s, {n: toks}, [[(n, n)]])[n], want, tol_of(dtype), f'{n} tokens at once')
            check(replay(s, {-n: toks}, [[(-n, 1)]] * n)[-n], want, tol_of(dtype), f'{n} tokens one by one')


@pytest.mark.parametrize('stack', sorted(STACKS))
def test_long_decoding(stack):
    cfg = STACKS[stack]
    toks = tokens_for(cfg, 330, 9)
    for dtype in ('float32', 'bfloat16'):
        w = weights_for(cfg, 15, dtype, toks)
        s = session_for(cfg, w, dtype)
        check_rows(replay(s, {'a': toks}, [[('a', 2)]] + [[('a', 1)]] * 328)['a'], toks, w, cfg, dtype, dtype)


# ------------------------------------------------------------------------------------------------ the options beside other ones
class DescribedModel(object):
    """An engine configuration and weights, served by a session like a model of the registry."""
    page_size = 64

    def __init__(self, config, w):
        self.config, self.w = config, w

    def build_stack_engine(self, dtype, num_blocks, num_slots, debug_taps=False, build_if_missing=False):
        from tensorrt_llm.runtime.stack import StackEngine
        return StackEngine(dict(self.config, dtype=dtype, num_blocks=num_blocks, num_slots=num_slots, debug_taps=int(debug_taps)), as_tensors(self.w))


def moe_keys(mlp):
    return {'layer.0.mlp': 'moe', 'layer.0.ff': mlp['expert']['ff'], 'layer.0.expert': 'relu2', 'layer.0.experts': mlp['router']['experts'],
            'layer.0.top': mlp['router']['top'], 'layer.0.route_score': 'sigmoid', 'layer.0.route_norm': 1, 'layer.0.shared_ff': mlp['shared']['ff']}


@pytest.mark.parametrize('width,mlp', [(96, moe(experts=4, top=4)), (128, moe(experts=4, top=4, ff=64, shared=128))])
@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_relu2_and_shared_experts_behind_a_sequential_block(dtype, width, mlp):
    """The same latent layer and mixture as pre-norm sublayers with a norm each: x <- x + mixer(n1 x), x <- x + ff(n2 x)."""
    from tensorrt_llm.runtime import RaggedGenerationSession
    cfg = make_config([layer(mlp=mlp)], width=width, side=0)
    w = random_weights(cfg, 41)
    w['l0.norm2'] = bf16_round(np.random.default_rng(1).standard_normal(width).astype(np.float32) * 0.2 + 1.0)
    m = cfg['layers'][0]['mixer']
    ec = dict(width=width, vocab=cfg['vocab'], num_layers=1, norm_eps=repr(1e-5), block='sequential', residual='hyper', streams=1,
              **{'layer.0.type': 'latent_attention', 'layer.0.rot_dim': 0, 'layer.0.sink': 1, 'layer.0.out_gate': 1,
                 **{'layer.0.' + k: m[k] for k in ('heads', 'dim', 'vdim', 'kv_rank', 'scale')}}, **moe_keys(mlp))
    toks = tokens_for(cfg, 90, 42)
    wf = as_f64(w)
    x = wf['embed'][toks]
    x = x + O.latent_attention(O.rms_norm(x, wf['l0.norm1'], 1e-5), wf, 'l0.mix.', m, 1e-5)
    x = x + O.moe_ff(O.rms_norm(x, wf['l0.norm2'], 1e-5), wf, 'l0.mlp.', mlp)
    want = O.rms_norm(x, wf['final.norm'], 1e-5) @ wf['head'].T
    s = RaggedGenerationSession(DescribedModel(ec, w), dtype=dtype, max_tokens=256)
    check(replay(s, {'a': toks}, [[('a', 80)]] + [[('a', 1)]] * 10)['a'], want, tol_of(dtype))


@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_grouped_query_attention_under_a_plain_residual(dtype):
    """Ordinary attention (no rotation) beside the mixture with its shared expert, on the one normed row."""
    from tensorrt_llm.runtime import RaggedGenerationSession
    mlp, W, H, G, D = moe(experts=3, top=3), 96, 4, 2, 16
    cfg = make_config([layer(mlp=mlp)], width=W, side=0)
    w = {k: v for k, v in random_weights(cfg, 43).items() if not k.startswith('l0.mix.')}
    rng = np.random.default_rng(2)
    for name, shape in (('q', (H * D, W)), ('k', (G * D, W)), ('v', (G * D, W)), ('o', (W, H * D)), ('g', (H, W))):
        w['l0.mix.' + name] = bf16_round(rng.standard_normal(shape).astype(np.float32) * 1.5 / shape[1] ** 0.5)
    ec = dict(width=W, vocab=cfg['vocab'], num_layers=1, norm_eps=repr(1e-5), block='parallel', residual='plain', embedding_norm=1, loop_input=0,
              **{'layer.0.type': 'attention', 'layer.0.heads': H, 'layer.0.kv_heads': G, 'layer.0.dim': D, 'layer.0.out_gate': 1,
                 'layer.0.scale': 0.25}, **moe_keys(mlp))
    toks = tokens_for(cfg, 90, 44)
    wf = as_f64(w)
    x = O.embed(toks, wf, 1e-5)
    h = O.rms_norm(x, wf['l0.norm1'], 1e-5)
    q, k, v = [(h @ wf['l0.mix.' + c].T).reshape(len(toks), -1, D) for c in 'qkv']
    gate = O.sigmoid(h @ wf['l0.mix.g'].T)
    ctx = np.concatenate([gate[:, a:a + 1] * (O.sink_softmax(q[:, a] @ k[:, a // 2].T * 0.25, -1e9) @ v[:, a // 2]) for a in range(H)], axis=1)
    x = x + ctx @ wf['l0.mix.o'].T + O.moe_ff(h, wf, 'l0.mlp.', mlp)
    want = O.rms_norm(x, wf['final.norm'], 1e-5) @ wf['head'].T
    s = RaggedGenerationSession(DescribedModel(ec, w), dtype=dtype, max_tokens=256)
    check(replay(s, {'a': toks}, [[('a', 80)]] + [[('a', 1)]] * 10)['a'], want, tol_of(dtype))


def test_descriptions_that_cannot_run_are_refused():
    from tensorrt_llm.runtime.stack import StackEngine
    cfg = make_config([layer(mlp=moe())])
    w = random_weights(cfg, 45)
    good = as_model(cfg, w).config.engine_config()
    good.update(dtype='float32', num_blocks=2, num_slots=1)
    for change in ({'block': 'sequential'}, {'loop_input': 1}, {'norm_groups': 3}, {'layer.0.mlp': 'gelu_gate'}, {'token_side': -1},
                   {'layer.0.expert': 'silu_gate'}, {'layer.0.top': 65, 'layer.0.experts': 70}):
        with pytest.raises(RuntimeError):
            StackEngine(dict(good, **change), as_tensors(w))
    with pytest.raises(RuntimeError, match='side.proj'):
        StackEngine(good, as_tensors({k: v for k, v in w.items() if k != 'l0.side.proj'}))


SMALL = make_config([layer(heads=2, mlp=moe(experts=4, top=2, ff=16, shared=24)), layer(heads=3, mlp=None), layer(heads=1, mlp=moe(experts=3, top=1, ff=20, shared=0))],
                    width=64, vocab=97, loop=(0, 2, 2), side=6)


def test_greedy_generation_through_the_scheduler():
    """Six prompts, four slots, 40 tokens per step: prompts are cut, requests queue, decoded tokens share steps with prompt portions.
    fp32 engine against the oracle's greedy continuation (recomputed from scratch for every token)."""
    from tensorrt_llm.runtime import SamplingConfig
    cfg = SMALL
    w = random_weights(cfg, seed=17)
    prompts = [tokens_for(cfg, n, 60 + n) for n in (70, 3, 45, 1, 90, 17)]
    s = session_for(cfg, w, 'float32', max_tokens=512, max_sequences=4, max_batch_tokens=40)
    outs = s.decode_batch(prompts, SamplingConfig(end_id=-1, pad_id=0), max_new_tokens=6)
    for p, o in zip(prompts, outs):
        assert o.tolist() == O.greedy(p, as_f64(w), cfg, 6)
    assert not s.live() and s.cache.blocks_manager.num_free_blocks() == s.num_blocks


def test_command_lines(tmp_path):
    """examples/sodudra/run.py generates from a checkpoint directory; bin/trace_run replays a recorded schedule from it."""
    from test_gpu_tolenex import write_checkpoint
    cfg = SMALL
    w = random_weights(cfg, seed=19)
    ck = str(tmp_path / 'ck')
    write_checkpoint(ck, cfg, w)
    prompt = tokens_for(cfg, 21, 70)
    np.save(tmp_path / 'in.npy', np.asarray(prompt, np.int32))
    run = os.path.join(ROOT, 'trtllm-llama_amd', 'examples', 'sodudra', 'run.py')
    subprocess.run([sys.executable, run, '--model_dir', ck, '--dtype', 'float32', '--input_tokens', str(tmp_path / 'in.npy'),
                    '--max_output_len', '5', '--output_npy', str(tmp_path / 'out.npy')], check=True, timeout=300)
    assert np.load(tmp_path / 'out.npy').reshape(-1)[len(prompt):].tolist() == O.greedy(prompt, as_f64(w), cfg, 5)
    a, b = tokens_for(cfg, 70, 71), tokens_for(cfg, 5, 72)
    steps = [{'step': 0, 'entries': [{'id': 'a', 'tokens': a[:66], 'want': [0, 65]}, {'id': 'b', 'tokens': b[:2], 'want': []}], 'end': []},
             {'step': 1, 'entries': [{'id': 'b', 'tokens': b[2:], 'want': [2]}], 'end': ['b']},
             {'step': 2, 'entries': [{'id': 'a', 'tokens': a[66:], 'want': [3]}], 'end': ['a']}]
    out = tmp_path / 'logits'
    r = subprocess.run([os.path.join(ROOT, 'bin', 'trace_run'), '--model', ck, '--dtype', 'float32', '--out', str(out), '--max-tokens', '192'],
                       input='\n'.join(json.dumps(s) for s in steps) + '\n', capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith('done')] == ['done 0', 'done 1', 'done 2']
    la, lb = O.logits(a, as_f64(w), cfg), O.logits(b, as_f64(w), cfg)
    check(np.fromfile(out / '0.f32', '<f4').reshape(2, -1), la[[0, 65]], F32_TOL)
    check(np.fromfile(out / '1.f32', '<f4').reshape(1, -1), lb[[4]], F32_TOL)
    check(np.fromfile(out / '2.f32', '<f4').reshape(1, -1), la[[69]], F32_TOL)
