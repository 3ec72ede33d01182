"""Sodudra: a decoder stack on one plain residual whose layers run their two sublayers side by side on one normed row,
x <- x + (mixer(n(x)) + ff(n(x))), starting from a normed embedding row.

  latent_attention   no positions: queries straight from the row, keys and values of every head expanded from one normed latent per
                     token; causal softmax whose denominator holds a per-head sink; a sigmoid gate per head on the output.  The cache
                     holds the latent; the engine runs the absorbed form
  moe                experts W_down relu(W_up h)^2; sigmoid scores, the `top` best chosen, weighted by their scores over the scores'
                     sum; a shared expert of the same form runs for every token

Behind every layer its token input lands: e = the layer's part of a per-token side embedding, y = W_proj (gelu_tanh(W_gate x) * e),
x <- x + n(y).  A range of layers may run several times in a row on the same weights (a cache per pass); each pass first adds a step
vector of its own.  Logits are scaled and soft-capped.

This class reads config.json and the safetensors file and describes the stack to the ragged engine (runtime/stack.py).  What the
design fixes lives here (which options the mixer and the router switch on, the experts' activation); every size and every other
constant is read from the configuration."""
import json
from typing import Dict

import numpy as np

from ..stack_model import PAGE_SIZE, StackModelForCausalLM, to_bf16_bits

MIXERS = ('latent_attention', )
MLP_KINDS = ('moe', )


class SodudraConfig(object):
    """config.json: architecture, vocab, width, norm.eps, logit_scale, logit_softcap, loop{start, stop, times} (absent: no loop),
    token_side{dim} (absent: none), layers[i].{type, mixer{heads, dim, vdim, kv_rank, scale}, mlp{kind, expert{ff},
    router{experts, top}, shared{ff}} | null}."""

    def __init__(self, d: Dict):
        self.raw = d
        self.vocab, self.width = int(d['vocab']), int(d['width'])
        self.norm_eps = float((d.get('norm') or {}).get('eps', 1e-6))
        self.logit_scale = float(1.0 if d.get('logit_scale') is None else d['logit_scale'])
        self.logit_softcap = float(d.get('logit_softcap') or 0.0)
        self.token_side = int((d.get('token_side') or {}).get('dim', 0))
        self.layers = d['layers']
        loop = d.get('loop') or {}
        self.loop = (int(loop.get('start', 0)), int(loop.get('stop', 0)), int(loop.get('times', 1)))
        for i, l in enumerate(self.layers):
            if l['type'] not in MIXERS:
                raise ValueError(f"layer {i}: mixer type {l['type']!r} is not one this design has {MIXERS}")
            mlp = l.get('mlp')
            if mlp is not None and mlp.get('kind', 'moe') not in MLP_KINDS:
                raise ValueError(f"layer {i}: feed-forward kind {mlp.get('kind')!r} {MLP_KINDS}")

    @staticmethod
    def from_json_file(path: str) -> 'SodudraConfig':
        with open(path) as f:
            return SodudraConfig(json.load(f))

    @property
    def looped(self) -> bool:
        return self.loop[1] > self.loop[0]

    def engine_config(self) -> Dict:
        c = dict(width=self.width, vocab=self.vocab, num_layers=len(self.layers), norm_groups=1, norm_eps=repr(self.norm_eps),
                 page_size=PAGE_SIZE, block='parallel', residual='plain', embedding_norm=1, loop_input=0, token_side=self.token_side,
                 logit_scale=repr(self.logit_scale), logit_softcap=repr(self.logit_softcap))
        if self.looped:
            c['loop_start'], c['loop_stop'], c['loop_times'] = self.loop
        for i, l in enumerate(self.layers):
            p, m = f'layer.{i}.', l['mixer']
            c[p + 'type'] = l['type']
            for k in ('heads', 'dim', 'vdim', 'kv_rank'):
                c[p + k] = int(m[k])
            c[p + 'scale'] = repr(float(m['scale']))
            c[p + 'rot_dim'], c[p + 'sink'], c[p + 'out_gate'] = 0, 1, 1
            mlp = l.get('mlp')
            if not mlp:
                c[p + 'ff'] = 0
                continue
            r = mlp['router']
            c[p + 'ff'], c[p + 'mlp'], c[p + 'expert'] = int(mlp['expert']['ff']), 'moe', 'relu2'
            c[p + 'experts'], c[p + 'top'] = int(r['experts']), int(r['top'])
            c[p + 'route_score'], c[p + 'route_norm'] = 'sigmoid', 1
            c[p + 'shared_ff'] = int((mlp.get('shared') or {}).get('ff', 0))
        return c


class SodudraForCausalLM(StackModelForCausalLM):
    architecture = 'Sodudra'
    config_class = SodudraConfig

    @classmethod
    def from_random(cls, config: Dict, seed: int = 0) -> 'SodudraForCausalLM':
        """Random bfloat16-valued weights of the configuration's shapes (benchmarks, examples)."""
        cfg = config if isinstance(config, SodudraConfig) else SodudraConfig(config)
        rng = np.random.default_rng(seed)
        t = {}

        def mat(name, *shape, s=1.0, mean=0.0):
            a = (rng.standard_normal(shape, dtype=np.float32) * s + mean).astype(np.float32)
            t[name] = (to_bf16_bits(a), 'bfloat16')

        W, S = cfg.width, cfg.token_side
        mat('embed', cfg.vocab, W)
        mat('embed.norm', W, s=0.1, mean=1.0)
        mat('head', cfg.vocab, W, s=W ** -0.5)
        mat('final.norm', W, s=0.1, mean=1.0)
        if cfg.looped:
            mat('loop.step', cfg.loop[2], W, s=0.1)
        if S:
            mat('side.embed', cfg.vocab, S * len(cfg.layers))
        for i, l in enumerate(cfg.layers):
            p, m = f'l{i}.', l['mixer']
            H, D, E, C = int(m['heads']), int(m['dim']), int(m['vdim']), int(m['kv_rank'])
            mat(p + 'norm1', W, s=0.1, mean=1.0)
            mat(p + 'mix.q', H * D, W, s=W ** -0.5)
            mat(p + 'mix.dkv', C, W, s=W ** -0.5)
            mat(p + 'mix.dkv.norm', C, s=0.1, mean=1.0)
            mat(p + 'mix.uk', H * D, C, s=C ** -0.5)
            mat(p + 'mix.uv', H * E, C, s=C ** -0.5)
            mat(p + 'mix.sink', H, s=0.5)
            mat(p + 'mix.g', H, W, s=W ** -0.5)
            mat(p + 'mix.o', W, H * E, s=(H * E) ** -0.5)
            if S:
                mat(p + 'side.gate', S, W, s=W ** -0.5)
                mat(p + 'side.proj', W, S, s=S ** -0.5)
                mat(p + 'side.norm', W, s=0.1, mean=0.3)
            mlp = l.get('mlp')
            if not mlp:
                continue
            ne = int(mlp['router']['experts'])
            kinds = [(f'e{e}.', int(mlp['expert']['ff'])) for e in range(ne)]
            if mlp.get('shared'):
                kinds.append(('shared.', int(mlp['shared']['ff'])))
            for n, F in kinds:
                mat(p + 'mlp.' + n + 'up', F, W, s=W ** -0.5)
                mat(p + 'mlp.' + n + 'down', W, F, s=F ** -0.5)
            mat(p + 'mlp.router', ne, W, s=2.0 * W ** -0.5)
        return cls(cfg, t)
