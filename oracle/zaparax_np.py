"""Plain NumPy statement of the Zaparax design: one function per mechanism.

Test infrastructure, never shipped.  Everything is float64, whole sequences at a time: one token after the other where the
mechanism is a recurrence or picks experts, whole score matrices where it is attention; no function is shared with the
product path.  `plant` names a mistake to put into the oracle itself (on the CPU), so that a test can see that a
comparison would notice it: 'window' (one token wider), 'sink' (left out), 'prev' (the bigram's previous token),
'conv' (one tap late), 'pass' (a looped layer's second pass goes on with the first one's state).
"""
import numpy as np

F = np.float64


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1.0 + w)


def embedding(tokens, table, scale, bigram=None, pairs=None, plant=None):
    """Scaled token rows plus a row of the bigram table per (previous, current) pair; the first token has a row of its own."""
    tokens = np.asarray(tokens, np.int64)
    x = table[tokens] * scale
    if bigram is not None:
        prev = np.roll(tokens, 1 if plant != 'prev' else 2)
        rows = (prev * bigram['mul_prev'] + tokens * bigram['mul_cur']) % bigram['buckets']
        rows[0] = bigram['buckets']
        x = x + pairs[rows]
    return x


def short_conv(x, w, b, plant=None):
    """silu of a causal convolution per channel.  x [T, C], w [C, taps] with the current token's tap last, b [C]."""
    T, taps = x.shape[0], w.shape[1]
    y = np.tile(b, (T, 1))
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j - (1 if plant == 'conv' else 0)
            if s >= 0:
                y[t] += w[:, j] * x[s]
    return silu(y)


def state_space(x, B, C, dt, A_log, D, S=None):
    """x [T, H, V], B and C [T, H, N], dt [T, H] -> y [T, H, V] and the state [H, N, V] behind the last token."""
    T, H, V = x.shape
    S = np.zeros((H, B.shape[2], V)) if S is None else S.copy()
    y = np.empty_like(x)
    for t in range(T):
        keep = np.exp(-np.exp(A_log) * dt[t])
        S = keep[:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        y[t] = np.sum(S * C[t][:, :, None], axis=1) + D[:, None] * x[t]
    return y, S


def mamba2(h, W, c, eps, plant=None, S=None, state_out=None):
    T, H, V, N, G = h.shape[0], c['heads'], c['vdim'], c['state'], c['groups']
    inner = H * V
    u = h @ W['in'].T
    z, xbc, dt = u[:, :inner], u[:, inner:2 * inner + 2 * G * N], u[:, 2 * inner + 2 * G * N:]
    xbc = short_conv(xbc, W['conv'], W['conv.b'], plant)
    group = np.arange(H) // (H // G)
    x = xbc[:, :inner].reshape(T, H, V)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)[:, group]
    C = xbc[:, inner + G * N:].reshape(T, G, N)[:, group]
    dt = np.logaddexp(0.0, dt + W['dt_bias'])
    y, S = state_space(x, B, C, dt, W['A_log'], W['D'], S)
    if state_out is not None:
        state_out.append(S)
    y = y.reshape(T, inner) * silu(z)
    y = rms(y.reshape(T, c['norm_groups'], -1), eps).reshape(T, inner) * W['norm']
    return y @ W['o'].T


def temperature(p, coef, every):
    return 1.0 + coef * np.log(np.floor((p + 1) / every) + 1.0)


def window_weights(scores, i, j, size, slope, softcap=None, sink=None, plant=None):
    """Softmax weights [T, T] of one head from its scaled scores: capped, distance taken off, window, sink in the denominator."""
    s = scores if softcap is None else softcap * np.tanh(scores / softcap)
    s = s - slope * (i - j)
    seen = (j <= i) & (i - j < size + (1 if plant == 'window' else 0))
    s = np.where(seen, s, -np.inf)
    m = s.max(axis=1, keepdims=True)
    if sink is not None and plant != 'sink':
        m = np.maximum(m, sink)
    e = np.exp(s - m)
    den = e.sum(axis=1, keepdims=True)
    if sink is not None and plant != 'sink':
        den = den + np.exp(sink - m)
    return e / den


def window_attention(h, W, c, eps, plant=None):
    T, H, G, D, V = h.shape[0], c['heads'], c['kv_heads'], c['dim'], c['vdim']
    q = rms((h @ W['q'].T + W['q.b']).reshape(T, H, D), eps)
    k = rms((h @ W['k'].T + W['k.b']).reshape(T, G, D), eps)
    v = (h @ W['v'].T + W['v.b']).reshape(T, G, V)
    p = np.arange(T)
    t = c.get('q_temp')
    if t:
        q = q * temperature(p, t['coef'], t['every'])[:, None, None]
    out = np.empty((T, H, V))
    for n in range(H):
        g = n // (H // G)
        w = window_weights((q[:, n] @ k[:, g].T) * c['scale'], p[:, None], p[None, :], c['mask']['size'], 2.0 ** (-8.0 * (n + 1) / H),
                           c.get('softcap'), W['sink'][n], plant)
        out[:, n] = w @ v[:, g]
    return out.reshape(T, H * V) @ W['o'].T


def gated(h, W):
    return (silu(h @ W['gate'].T) * (h @ W['up'].T)) @ W['down'].T


def choose(h, W, r):
    """Per token the chosen experts (best first) and their weights."""
    z = h @ W['router'].T
    s = np.exp(z - z.max(axis=1, keepdims=True))
    s /= s.sum(axis=1, keepdims=True)
    ids = np.argsort(-(s + W['correction']), axis=1, kind='stable')[:, :r['top']]
    return ids, np.take_along_axis(s, ids, axis=1)


def experts(h, W, c):
    """Mixture of experts; those past the last matrix give their input back."""
    r = c['router']
    ids, wt = choose(h, W, r)
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(ids[t], wt[t]):
            y[t] += w * (gated(h[t], sub(W, f'e{e}.')) if e < r['experts'] else h[t])
    if c.get('shared'):
        y += sigmoid(h @ W['shared.sg'].T) * gated(h, sub(W, 'shared.'))
    return y


def sub(W, prefix):
    return {n[len(prefix):]: a for n, a in W.items() if n.startswith(prefix)}


def layer_runs(cfg):
    """The layers in the order they run."""
    n, loop = len(cfg['layers']), cfg.get('loop')
    if not loop:
        return list(range(n))
    a, b = loop['start'], loop['stop']
    return list(range(a)) + list(range(a, b)) * loop['times'] + list(range(b, n))


def forward(cfg, W, tokens, layers_out=None, plant=None):
    """Logits [T, vocab] of a whole sequence.  cfg: the parsed config.json; W: tensor name -> array."""
    W = {n: np.asarray(a, F) for n, a in W.items()}
    eps, emb = cfg['norm']['eps'], cfg['embedding']
    x = embedding(tokens, W['embed'], emb['scale'], emb.get('bigram'), W.get('bigram'), plant)
    left = {}
    for i in layer_runs(cfg):
        L, p = cfg['layers'][i], f'l{i}.'
        mix, h = sub(W, p + 'mix.'), norm(x, W[p + 'norm1'], eps)
        if L['type'] == 'mamba2':
            got = []
            y = mamba2(h, mix, L['mixer'], eps, plant, left.get(i) if plant == 'pass' else None, got)
            left[i] = got[0]
        else:
            y = window_attention(h, mix, L['mixer'], eps, plant)
        x = x + norm(y, W[p + 'norm1b'], eps)
        if L['mlp'] is not None:
            h, mlp = norm(x, W[p + 'norm2'], eps), sub(W, p + 'mlp.')
            y = experts(h, mlp, L['mlp']) if L['mlp']['kind'] == 'moe' else gated(h, mlp)
            x = x + norm(y, W[p + 'norm2b'], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return norm(x, W['final.norm'], eps) @ W['head'].T
