"""Plain float64 numpy statement of the Sodudra design, one function per mechanism.  Test infrastructure only: slow, whole
sequences, no cache, no batching - the product (the stack engine) never touches it and shares no code with it.

Sodudra is a decoder stack on one residual stream whose layers run their two sublayers side by side on ONE normed row:
  x <- n_e(embed[token]);  per layer  h = n(x),  x <- x + (mixer(h) + ff(h)),  then the layer's token input is added.
  mixer       latent attention without positions: queries straight from h, keys and values of every head expanded from one normed
              latent per token, causal softmax whose denominator holds a per-head sink, a sigmoid gate per head on the output;
  ff          a routed mixture of experts W_down relu(W_up h)^2: sigmoid scores, the best `top` chosen, their scores divided by their
              sum as weights; a shared expert of the same form runs for every token;
  token input e = the layer's part of a per-token side embedding, y = W_proj (gelu_tanh(W_gate x) * e), x <- x + n(y);
  loop        a range of layers runs several times in a row on the same weights, every pass after adding its own step vector;
  output      logits = cap * tanh(scale * W_head n(x) / cap).

Notation: n tokens, width W.  `w` is a dict name -> float64 array with the checkpoint's names; `cfg` is the parsed config.json."""
import math

import numpy as np

# A test may ask how much rounding of the activations moves a result: inside `with rounding(fn):` every projection's output, every
# norm's output (the embedding's, which is the residual, stays), attention weights and the experts' hidden activations pass
# through fn.  It is an estimate of a row's conditioning, not a model of any engine.
_round = None


class rounding(object):
    def __init__(self, fn):
        self.fn = fn

    def __enter__(self):
        global _round
        self.old, _round = _round, self.fn

    def __exit__(self, *exc):
        global _round
        _round = self.old


def _r(x):
    return x if _round is None else _round(x)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z):
    return np.maximum(z, 0.0) ** 2


def rms_norm(x, weight, eps):
    """x / sqrt(mean(x^2) + eps) * weight over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


# ------------------------------------------------------------------------------------------------ ends of the stack
def embed(tokens, w, eps):
    """The normed embedding row: the residual starts from it."""
    return rms_norm(w['embed'][np.asarray(tokens)], w['embed.norm'], eps)


def head(x, w, cfg):
    """Scaled, soft-capped logits of the normed residual."""
    z = _r(rms_norm(x, w['final.norm'], float(cfg['norm']['eps']))) @ w['head'].T * float(cfg.get('logit_scale', 1.0))
    cap = float(cfg.get('logit_softcap') or 0.0)
    return cap * np.tanh(z / cap) if cap else z


# ------------------------------------------------------------------------------------------------ latent attention
def sink_softmax(scores, sink):
    """Causal row-wise softmax of scores [n, n] whose denominator also holds exp(sink)."""
    n = scores.shape[0]
    vis = np.arange(n)[None, :] <= np.arange(n)[:, None]
    s = np.where(vis, scores, -np.inf)
    top = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - top)
    return _r(e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - top)))


def latent_attention(h, w, p, m, eps):
    """Mixer 'latent_attention'.  h [n, W] -> [n, W]."""
    n = h.shape[0]
    H, D, E = int(m['heads']), int(m['dim']), int(m['vdim'])
    q = _r(h @ w[p + 'q'].T).reshape(n, H, D)
    c = _r(rms_norm(_r(h @ w[p + 'dkv'].T), w[p + 'dkv.norm'], eps))
    k = (c @ w[p + 'uk'].T).reshape(n, H, D)
    v = (c @ w[p + 'uv'].T).reshape(n, H, E)
    gate = sigmoid(_r(h @ w[p + 'g'].T))
    out = np.zeros((n, H, E))
    for a in range(H):
        prob = sink_softmax(q[:, a] @ k[:, a].T * float(m['scale']), float(w[p + 'sink'][a]))
        out[:, a] = _r(gate[:, a:a + 1] * (prob @ v[:, a]))
    return out.reshape(n, H * E) @ w[p + 'o'].T


# ------------------------------------------------------------------------------------------------ feed-forward
def expert(h, w, p):
    return _r(relu_squared(_r(h @ w[p + 'up'].T))) @ w[p + 'down'].T


def route(h, w, p, r):
    """-> (chosen [n, top] expert numbers, weights [n, top] that sum to one)."""
    s = sigmoid(h @ w[p + 'router'].T)
    chosen = np.argsort(-s, axis=-1, kind='stable')[:, :int(r['top'])]
    g = np.take_along_axis(s, chosen, axis=-1)
    return chosen, g / (g.sum(axis=-1, keepdims=True) + 1e-20)


def moe_ff(h, w, p, mlp):
    chosen, weights = route(h, w, p, mlp['router'])
    out = np.zeros((h.shape[0], h.shape[1]))
    for e in range(int(mlp['router']['experts'])):
        rows, place = np.nonzero(chosen == e)
        if len(rows):
            out[rows] += weights[rows, place][:, None] * expert(h[rows], w, f'{p}e{e}.')
    if mlp.get('shared'):
        out += expert(h, w, p + 'shared.')
    return out


# ------------------------------------------------------------------------------------------------ token input of a layer
def token_side(x, tokens, w, cfg, i):
    """The addition layer i makes from the side embedding of its tokens."""
    p, d = f'l{i}.side.', int(cfg['token_side']['dim'])
    e = w['side.embed'][np.asarray(tokens)][:, i * d:(i + 1) * d]
    y = _r(gelu_tanh(_r(_r(x) @ w[p + 'gate'].T)) * e) @ w[p + 'proj'].T
    return rms_norm(y, w[p + 'norm'], float(cfg['norm']['eps']))


# ------------------------------------------------------------------------------------------------ the stack
def execution(cfg):
    """[(layer, pass, enters a pass)] in the order they run."""
    L, loop = len(cfg['layers']), cfg.get('loop')
    if not loop:
        return [(i, 0, False) for i in range(L)]
    a, b, times = int(loop['start']), int(loop['stop']), int(loop['times'])
    runs = [(i, 0, False) for i in range(a)]
    for t in range(times):
        runs += [(i, t, i == a) for i in range(a, b)]
    return runs + [(i, 0, False) for i in range(b, L)]


def layer_forward(x, tokens, w, cfg, i):
    l, eps, p = cfg['layers'][i], float(cfg['norm']['eps']), f'l{i}.'
    h = _r(rms_norm(x, w[p + 'norm1'], eps))
    add = latent_attention(h, w, p + 'mix.', l['mixer'], eps)
    if l.get('mlp'):
        add = add + moe_ff(h, w, p + 'mlp.', l['mlp'])
    x = x + add
    if cfg.get('token_side'):
        x = x + token_side(x, tokens, w, cfg, i)
    return x


def forward(tokens, w, cfg, return_layers=False):
    """tokens [n] -> logits [n, vocab] (and the residual stream behind every layer run, [runs, n, W])."""
    x = embed(tokens, w, float(cfg['norm']['eps']))
    taps = []
    for i, t, enters in execution(cfg):
        if enters:
            x = x + w['loop.step'][t]
        x = layer_forward(x, tokens, w, cfg, i)
        taps.append(x)
    logits = head(x, w, cfg)
    return (logits, np.stack(taps)) if return_layers else logits


def logits(tokens, w, cfg):
    return forward(tokens, w, cfg)


def greedy(prompt, w, cfg, n_new):
    """The greedy continuation, recomputed from scratch for every token."""
    toks, out = list(prompt), []
    for _ in range(n_new):
        nxt = int(np.argmax(forward(toks, w, cfg)[-1]))
        out.append(nxt)
        toks.append(nxt)
    return out
