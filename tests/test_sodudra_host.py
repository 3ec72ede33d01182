"""Host-side pieces of the Sodudra design that need no GPU: the configuration reader and the registry, the random-weight maker's
tensor list, and the oracle's own mechanisms against closed forms and against a second way of computing them."""
import math

import numpy as np
import pytest

from oracle import sodudra_oracle as O
from sodudra_cases import decisive_router, layer, make_config, moe, random_weights, routing_margin
from tolenex_cases import as_f64


def test_registry_picks_the_class_by_config():
    from tensorrt_llm.models import MODEL_REGISTRY, SodudraForCausalLM, model_class_for
    assert model_class_for({'architecture': 'Sodudra'}) is SodudraForCausalLM
    assert {'Sodudra', 'Narurax', 'Rofozen', 'Vetipel', 'Tolenex'} <= set(MODEL_REGISTRY)


def test_config_reader_takes_every_size_from_the_file():
    from tensorrt_llm.models import SodudraConfig
    cfg = make_config([layer(heads=7, dim=10, vdim=14, kv_rank=50, scale=0.321, mlp=moe(experts=9, top=4, ff=17, shared=33)),
                       layer(heads=1, dim=3, vdim=5, kv_rank=8, mlp=None), layer(mlp=moe(shared=0))],
                      width=140, vocab=1001, eps=3e-6, loop=(1, 3, 4), side=20, logit_scale=0.3, softcap=7.5)
    c = SodudraConfig(cfg).engine_config()
    assert (c['width'], c['vocab'], c['num_layers'], c['block'], c['residual']) == (140, 1001, 3, 'parallel', 'plain')
    assert (c['embedding_norm'], c['loop_input'], c['token_side']) == (1, 0, 20)
    assert (float(c['norm_eps']), float(c['logit_scale']), float(c['logit_softcap'])) == (3e-6, 0.3, 7.5)
    assert (c['loop_start'], c['loop_stop'], c['loop_times']) == (1, 3, 4)
    assert [c['layer.0.' + k] for k in ('type', 'heads', 'dim', 'vdim', 'kv_rank', 'rot_dim', 'sink', 'out_gate')] == [
        'latent_attention', 7, 10, 14, 50, 0, 1, 1]
    assert float(c['layer.0.scale']) == 0.321
    assert [c['layer.0.' + k] for k in ('mlp', 'expert', 'ff', 'experts', 'top', 'shared_ff', 'route_score', 'route_norm')] == [
        'moe', 'relu2', 17, 9, 4, 33, 'sigmoid', 1]
    assert c['layer.1.ff'] == 0 and c['layer.2.shared_ff'] == 0
    plain = {k: v for k, v in make_config([layer()], side=0).items() if k not in ('logit_scale', 'logit_softcap')}
    c = SodudraConfig(plain).engine_config()
    assert 'loop_start' not in c and c['token_side'] == 0 and float(c['logit_scale']) == 1.0 and float(c['logit_softcap']) == 0.0
    with pytest.raises(ValueError):
        SodudraConfig(make_config([{'type': 'mamba2', 'mixer': {}, 'mlp': None}]))
    with pytest.raises(ValueError):
        SodudraConfig(make_config([layer(mlp={'kind': 'dense', 'ff': 8})]))


def test_random_weight_maker_names_what_the_tests_generator_names():
    """Two generators written apart (the product's, for benchmarks; the tests') must agree on names and shapes."""
    from tensorrt_llm.models import SodudraForCausalLM
    for kw in (dict(loop=(1, 2, 3)), dict(side=0)):
        cfg = make_config([layer(mlp=moe()), layer(heads=2, mlp=moe(shared=0)), layer()], **kw)
        ours = random_weights(cfg, 1)
        theirs = SodudraForCausalLM.from_random(cfg, seed=2).tensors
        assert {k: v.shape for k, v in ours.items()} == {k: a.shape for k, (a, _) in theirs.items()}


def test_execution_order_of_a_loop():
    cfg = make_config([layer()] * 4, loop=(1, 3, 2))
    assert O.execution(cfg) == [(0, 0, False), (1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False), (3, 0, False)]
    assert O.execution(make_config([layer()] * 2, loop=(0, 2, 1))) == [(0, 0, True), (1, 0, False)]
    assert O.execution(make_config([layer()] * 2)) == [(0, 0, False), (1, 0, False)]


def test_every_pass_adds_its_step_once_and_nothing_else():
    """A loop of t passes is the unrolled stack with each pass's step added by hand."""
    cfg = make_config([layer(), layer(heads=2)], loop=(0, 2, 2))
    w = as_f64(random_weights(cfg, 4))
    toks = [5, 9, 2]
    x = O.embed(toks, w, cfg['norm']['eps'])
    for t in range(2):
        x = x + w['loop.step'][t]
        for i in range(2):
            x = O.layer_forward(x, toks, w, cfg, i)
    assert np.allclose(O.forward(toks, w, cfg), O.head(x, w, cfg), rtol=1e-12, atol=1e-12)


def test_both_sublayers_read_the_same_row():
    cfg = make_config([layer(mlp=moe())], side=0)
    w = as_f64(random_weights(cfg, 5))
    x = np.random.default_rng(1).standard_normal((4, 96))
    h = O.rms_norm(x, w['l0.norm1'], 1e-5)
    want = x + O.latent_attention(h, w, 'l0.mix.', cfg['layers'][0]['mixer'], 1e-5) + O.moe_ff(h, w, 'l0.mlp.', cfg['layers'][0]['mlp'])
    assert np.allclose(O.layer_forward(x, [1, 2, 3, 4], w, cfg, 0), want, rtol=1e-12, atol=1e-12)


def test_a_sink_takes_its_share_and_a_gate_scales_a_head():
    """One token: the only key is the token itself, so head a's output is sigmoid(g_a) v e^s / (e^s + e^sink)."""
    cfg = make_config([layer(heads=2, dim=4, vdim=3, kv_rank=6)], width=8, vocab=11, side=0)
    w = as_f64(random_weights(cfg, 3))
    m, p = cfg['layers'][0]['mixer'], 'l0.mix.'
    h = np.random.default_rng(0).standard_normal((1, 8))
    q = (h @ w[p + 'q'].T).reshape(2, 4)
    c = O.rms_norm(h @ w[p + 'dkv'].T, w[p + 'dkv.norm'], 1e-5)[0]
    heads = []
    for a in range(2):
        s = q[a] @ (w[p + 'uk'][a * 4:(a + 1) * 4] @ c) * m['scale']
        share = math.exp(s) / (math.exp(s) + math.exp(w[p + 'sink'][a]))
        heads.append(share * (w[p + 'uv'][a * 3:(a + 1) * 3] @ c) / (1.0 + math.exp(-float(h[0] @ w[p + 'g'][a]))))
    assert np.allclose(O.latent_attention(h, w, p, m, 1e-5)[0], np.concatenate(heads) @ w[p + 'o'].T, rtol=1e-12, atol=1e-12)


def test_latent_attention_equals_its_absorbed_form():
    """Scores through W_uk^T q against the latent, the gate on the weighted sum of latents, values expanded last: the same function."""
    cfg = make_config([layer(heads=3, dim=6, vdim=5, kv_rank=10)], width=16, vocab=11, side=0)
    w = as_f64(random_weights(cfg, 5))
    m, p = cfg['layers'][0]['mixer'], 'l0.mix.'
    n, H, D, E = 9, 3, 6, 5
    h = np.random.default_rng(2).standard_normal((n, 16))
    q = (h @ w[p + 'q'].T).reshape(n, H, D)
    c = O.rms_norm(h @ w[p + 'dkv'].T, w[p + 'dkv.norm'], 1e-5)
    gate = O.sigmoid(h @ w[p + 'g'].T)
    out = np.zeros((n, H, E))
    for a in range(H):
        s = np.where(np.tril(np.ones((n, n), bool)), (q[:, a] @ w[p + 'uk'][a * D:(a + 1) * D]) @ c.T * m['scale'], -np.inf)
        e = np.exp(s)
        lat = (e / (e.sum(axis=1, keepdims=True) + np.exp(w[p + 'sink'][a]))) @ c * gate[:, a:a + 1]
        out[:, a] = lat @ w[p + 'uv'][a * E:(a + 1) * E].T
    assert np.allclose(O.latent_attention(h, w, p, m, 1e-5), out.reshape(n, H * E) @ w[p + 'o'].T, rtol=1e-10, atol=1e-12)


def test_router_weights_are_the_chosen_scores_over_their_sum():
    w = {'router': np.zeros((4, 3))}
    w['router'][:, 0] = [math.log(s / (1 - s)) for s in (0.4, 0.3, 0.9, 0.1)]
    chosen, weights = O.route(np.array([[1.0, 0.0, 0.0]]), w, '', {'experts': 4, 'top': 2})
    assert chosen[0].tolist() == [2, 0] and np.allclose(weights[0], [0.9 / 1.3, 0.4 / 1.3])
    chosen, weights = O.route(np.array([[1.0, 0.0, 0.0]]), w, '', {'experts': 4, 'top': 1})
    assert chosen[0].tolist() == [2] and np.allclose(weights, 1.0)


def test_mixture_against_a_loop_over_tokens_with_the_shared_expert_unweighted():
    cfg = make_config([layer(mlp=moe(experts=5, top=3, ff=7, shared=11))], width=16)
    w = as_f64(random_weights(cfg, 6))
    h = np.random.default_rng(3).standard_normal((6, 16))
    chosen, weights = O.route(h, w, 'l0.mlp.', cfg['layers'][0]['mlp']['router'])
    want = np.zeros((6, 16))
    for t in range(6):
        for e, g in zip(chosen[t], weights[t]):
            want[t] += g * (np.maximum(w[f'l0.mlp.e{e}.up'] @ h[t], 0) ** 2 @ w[f'l0.mlp.e{e}.down'].T)
        want[t] += np.maximum(w['l0.mlp.shared.up'] @ h[t], 0) ** 2 @ w['l0.mlp.shared.down'].T
    assert np.allclose(O.moe_ff(h, w, 'l0.mlp.', cfg['layers'][0]['mlp']), want, rtol=1e-12, atol=1e-12)


def test_a_layer_reads_its_own_part_of_the_side_embedding():
    cfg = make_config([layer(), layer(), layer()], side=4)
    w = as_f64(random_weights(cfg, 7))
    x = np.random.default_rng(4).standard_normal((2, 96))
    base = [O.token_side(x, [3, 8], w, cfg, i) for i in range(3)]
    w2 = dict(w, **{'side.embed': w['side.embed'].copy()})
    w2['side.embed'][8, 4:8] *= -1.5   # token 8, layer 1's part
    moved = [np.abs(O.token_side(x, [3, 8], w2, cfg, i) - base[i]).max(axis=1) for i in range(3)]
    assert moved[0].max() == 0 and moved[2].max() == 0 and moved[1][0] == 0 and moved[1][1] > 1e-3
    # the norm behind it makes its size that of the norm's weight, whatever the gate's
    y = base[1] / w['l1.side.norm']
    assert np.allclose(np.mean(y * y, axis=1), 1.0, atol=1e-2)


def test_logits_are_scaled_before_the_cap():
    cfg = make_config([layer()], logit_scale=0.25, softcap=3.0)
    w = as_f64(random_weights(cfg, 8))
    x = np.random.default_rng(5).standard_normal((2, 96))
    z = O.rms_norm(x, w['final.norm'], 1e-5) @ w['head'].T
    assert np.allclose(O.head(x, w, cfg), 3.0 * np.tanh(0.25 * z / 3.0))
    assert np.allclose(O.head(x, w, dict(cfg, logit_softcap=None, logit_scale=1.0)), z)


def test_rigged_routers_are_decisive():
    cfg = make_config([layer(mlp=moe()), layer(mlp=moe(experts=5, top=3))], loop=(0, 1, 2))
    w = decisive_router(cfg, random_weights(cfg, 9), 9)
    assert routing_margin(cfg, w, list(range(40))) > 0.2
