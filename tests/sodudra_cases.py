"""Small Sodudra configurations and random weights for the tests (own generator: nothing of the product's random-weight code)."""
import numpy as np

from tolenex_cases import bf16_round


def moe(experts=6, top=2, ff=24, shared=40):
    m = {'kind': 'moe', 'expert': {'ff': ff}, 'router': {'experts': experts, 'top': top}}
    if shared:
        m['shared'] = {'ff': shared}
    return m


def layer(heads=3, dim=16, vdim=24, kv_rank=40, scale=None, mlp=None):
    m = {'heads': heads, 'dim': dim, 'vdim': vdim, 'kv_rank': kv_rank, 'scale': 1.5 / dim ** 0.5 if scale is None else scale}
    return {'type': 'latent_attention', 'mixer': m, 'mlp': mlp}


def make_config(layers, width=96, vocab=211, eps=1e-5, loop=None, side=12, logit_scale=0.75, softcap=11.0):
    cfg = {'architecture': 'Sodudra', 'vocab': vocab, 'width': width, 'norm': {'eps': eps}, 'layers': layers,
           'logit_scale': logit_scale, 'logit_softcap': softcap}
    if side:
        cfg['token_side'] = {'dim': side}
    if loop:
        cfg['loop'] = {'start': loop[0], 'stop': loop[1], 'times': loop[2]}
    return cfg


def random_weights(cfg, seed=0):
    """name -> fp32 array of bfloat16-representable values, sized by cfg; scaled so that scores, gates and logits are O(1)."""
    rng = np.random.default_rng(seed)
    W, w = cfg['width'], {}

    def put(name, *shape, std=1.0, mean=0.0):
        w[name] = bf16_round(rng.standard_normal(shape).astype(np.float32) * std + mean)

    put('embed', cfg['vocab'], W, std=2.5)
    put('embed.norm', W, std=0.2, mean=1.0)
    put('head', cfg['vocab'], W, std=5.0 / W ** 0.5)
    put('final.norm', W, std=0.2, mean=1.0)
    if cfg.get('loop'):
        put('loop.step', cfg['loop']['times'], W, std=0.5)
    side = int((cfg.get('token_side') or {}).get('dim', 0))
    if side:
        put('side.embed', cfg['vocab'], side * len(cfg['layers']))
    for i, l in enumerate(cfg['layers']):
        p, m = f'l{i}.', l['mixer']
        H, D, E, C = m['heads'], m['dim'], m['vdim'], m['kv_rank']
        put(p + 'norm1', W, std=0.2, mean=1.0)
        put(p + 'mix.q', H * D, W, std=1.5 / W ** 0.5)
        put(p + 'mix.dkv', C, W, std=1.5 / W ** 0.5)
        put(p + 'mix.dkv.norm', C, std=0.2, mean=1.0)
        put(p + 'mix.uk', H * D, C, std=1.5 / C ** 0.5)
        put(p + 'mix.uv', H * E, C, std=2.0 / C ** 0.5)
        put(p + 'mix.sink', H, std=1.0, mean=1.0)
        put(p + 'mix.g', H, W, std=1.5 / W ** 0.5)
        put(p + 'mix.o', W, H * E, std=2.0 / (H * E) ** 0.5)
        if side:
            put(p + 'side.gate', side, W, std=1.0 / W ** 0.5)
            put(p + 'side.proj', W, side, std=1.0 / side ** 0.5)
            put(p + 'side.norm', W, std=0.1, mean=0.5)
        mlp = l.get('mlp')
        if not mlp:
            continue
        parts = [(f'e{e}.', mlp['expert']['ff']) for e in range(mlp['router']['experts'])]
        if mlp.get('shared'):
            parts.append(('shared.', mlp['shared']['ff']))
        for name, F in parts:
            put(p + 'mlp.' + name + 'up', F, W, std=1.0 / W ** 0.5)
            put(p + 'mlp.' + name + 'down', W, F, std=1.0 / F ** 0.5)
        put(p + 'mlp.router', mlp['router']['experts'], W, std=1.5 / W ** 0.5)
    return w


def as_model(cfg, w):
    """The product's model object over these weights (bfloat16 bit patterns, as a checkpoint reader would deliver them)."""
    from tensorrt_llm.models.sodudra.model import SodudraConfig, SodudraForCausalLM
    return SodudraForCausalLM(SodudraConfig(cfg), as_tensors(w))


def as_tensors(w):
    return {k: ((np.ascontiguousarray(v, np.float32).view(np.uint32) >> 16).astype(np.uint16).reshape(v.shape), 'bfloat16') for k, v in w.items()}


def decisive_router(cfg, w, seed=0, gain=10.0):
    """Rewrites w so that no router decision is a close call (for the bfloat16 engine, whose rounding moves scores by a percent):
    the last channels of the residual are reserved - nothing behind the embedding writes to them, so they hold what the embedding put
    there, a per-token ranking of the experts (all values <= 0, so that no score saturates) - and every router reads nothing but its
    own channel of them.  Scores of neighbouring ranks then differ by a factor."""
    rng = np.random.default_rng(seed)
    ne = max(l['mlp']['router']['experts'] for l in cfg['layers'] if l.get('mlp'))
    for k in w:
        if k.endswith('mix.o') or k.endswith('.down'):
            w[k][-ne:, :] = 0.0
        if k.endswith('side.norm'):
            w[k][-ne:] = 0.0
        if k.endswith('norm1') or k == 'embed.norm':
            w[k][-ne:] = 1.0
        if k == 'loop.step':
            w[k][:, -ne:] = 0.0
    w['embed'][:, -ne:] = -np.stack([rng.permutation(ne) for _ in range(cfg['vocab'])]).astype(np.float32)
    for i, l in enumerate(cfg['layers']):
        if not l.get('mlp'):
            continue
        n = l['mlp']['router']['experts']
        r = np.zeros_like(w[f'l{i}.mlp.router'])
        r[np.arange(n), r.shape[1] - ne + np.arange(n)] = gain
        w[f'l{i}.mlp.router'] = r
    return w


def routing_margin(cfg, w, toks):
    """The smallest relative gap (a - b) / (a + b), over tokens and routed layer runs, between the last chosen score and the first
    one left out, on the float64 oracle: a model whose margin is tiny would make a test rest on a close call."""
    from oracle import sodudra_oracle as O
    wf = {k: v.astype(np.float64) for k, v in w.items()}
    eps = cfg['norm']['eps']
    x = O.embed(toks, wf, eps)
    worst = np.inf
    for i, t, enters in O.execution(cfg):
        if enters:
            x = x + wf['loop.step'][t]
        mlp = cfg['layers'][i].get('mlp')
        if mlp and mlp['router']['top'] < mlp['router']['experts']:
            h = O.rms_norm(x, wf[f'l{i}.norm1'], eps)
            s = np.sort(O.sigmoid(h @ wf[f'l{i}.mlp.router'].T), axis=-1)[:, ::-1]
            a, b = s[:, mlp['router']['top'] - 1], s[:, mlp['router']['top']]
            worst = min(worst, ((a - b) / (a + b)).min())
        x = O.layer_forward(x, toks, wf, cfg, i)
    return worst
