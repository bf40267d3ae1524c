"""Plain NumPy statement of the layered-mixer models (architecture "Vomotar"): one function per mechanism.

Test infrastructure, never shipped.  Everything is float64, one token after the other where the mechanism is a
recurrence, whole score matrices where it is attention; no function is shared with the product path.
`plant` arguments let a test put a mistake into the oracle itself (on the CPU) and see that a comparison would
notice it.
"""
import numpy as np

F = np.float64


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def group_norm(x, w, groups, eps):
    """Rows of x cut into `groups` equal runs, each over its own root mean square; times w."""
    y = rms(x.reshape(x.shape[:-1] + (groups, x.shape[-1] // groups)), eps)
    return y.reshape(x.shape) * w


def causal_conv_silu(x, w):
    """Depthwise: y[t, c] = silu(sum_j w[c, j] x[t - (J - 1) + j, c]), zeros ahead of the sequence.  x [T, C], w [C, J]."""
    J = w.shape[1]
    xp = np.concatenate([np.zeros((J - 1, x.shape[1])), x], axis=0)
    y = sum(w[:, j] * xp[j:j + x.shape[0]] for j in range(J))
    return silu(y)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """q, k, g [T, H, D], v [T, H, V], beta [T, H] -> o [T, H, V], S [H, D, V]."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]))
    o = np.empty(v.shape)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum('hdv,hd->hv', S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum('hdv,hd->hv', S, q[t])
    return o, S


def channel_delta(h, W, c, eps):
    """Gated delta rule with a decay per key channel.  W: name -> array (the part behind '.mix.'); c: sizes."""
    T = h.shape[0]
    H, KH, D, V = c['heads'], c['kv_heads'], c['dim'], c['vdim']
    q = causal_conv_silu(h @ W['q'].T, W['q.conv']).reshape(T, KH, D)
    k = causal_conv_silu(h @ W['k'].T, W['k.conv']).reshape(T, KH, D)
    v = causal_conv_silu(h @ W['v'].T, W['v.conv']).reshape(T, H, V)
    pick = np.arange(H) // (H // KH)
    q, k = (unit(q) * D ** -0.5)[:, pick], unit(k)[:, pick]
    beta = sigmoid(h @ W['b'].T)
    a = ((h @ W['a1'].T) @ W['a2'].T + W['dt_bias']).reshape(T, H, D)
    g = np.exp(-np.exp(W['A_log'])[:, None] * softplus(a))
    o, _ = delta_rule(q, k, v, g, beta)
    gate = sigmoid((h @ W['g1'].T) @ W['g2'].T)
    return (rms(o, eps) * W['norm']).reshape(T, H * V) * gate @ W['o'].T


def chunk_attention(h, W, c, eps, plant=None):
    """Softmax attention without rotation, keys of the query's own chunk only, logarithmic distance penalty."""
    T = h.shape[0]
    H, G, D, V = c['heads'], c['kv_heads'], c['dim'], c['vdim']
    size = c['mask']['size']
    q = (h @ W['q'].T).reshape(T, H, D)
    k = (h @ W['k'].T).reshape(T, G, D)
    v = rms((h @ W['v'].T).reshape(T, G, V), eps)
    pick = np.arange(H) // (H // G)
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    shift = 1 if plant == 'edge' else 0
    seen = (j <= i) & ((i + shift) // size == (j + shift) // size)
    out = np.empty((T, H, V))
    for n in range(H):
        s = (q[:, n] @ k[:, pick[n]].T) * c['scale'] - W['r1'][n] * np.log1p(W['r2'][n] * np.maximum(i - j, 0))
        s = np.where(seen, s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, n] = (p / p.sum(axis=1, keepdims=True)) @ v[:, pick[n]]
    return out.reshape(T, H * V) @ W['o'].T


def rotate_half(x, base, dims, pos0=0):
    """x [T, H, D]: pairs (i, i + dims / 2) of the first `dims` dimensions turned by p * base^(-2 i / dims)."""
    half = dims // 2
    p = np.arange(x.shape[0]) + pos0
    ang = p[:, None] * base ** (-2.0 * np.arange(half) / dims)
    cs, sn = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    u, w = x[..., :half], x[..., half:dims]
    return np.concatenate([u * cs - w * sn, w * cs + u * sn, x[..., dims:]], axis=-1)


def retention(h, W, c, eps):
    """Linear attention with one fixed decay per head; gated, normed per head without weight."""
    T = h.shape[0]
    H, D, V = c['heads'], c['dim'], c['vdim']
    q = rotate_half((h @ W['q'].T).reshape(T, H, D), c['rot']['base'], c['rot']['dims'])
    k = rotate_half((h @ W['k'].T).reshape(T, H, D), c['rot']['base'], c['rot']['dims']) * D ** -0.5
    v = (h @ W['v'].T).reshape(T, H, V)
    dec = np.asarray(c['decay'], F)[:, None, None]
    S = np.zeros((H, D, V))
    o = np.empty((T, H, V))
    for t in range(T):
        S = dec * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum('hdv,hd->hv', S, q[t])
    return (rms(o, eps).reshape(T, H * V) * silu(h @ W['g'].T)) @ W['o'].T


def sub(W, prefix):
    return {n[len(prefix):]: a for n, a in W.items() if n.startswith(prefix)}


def parallel(h, W, c, eps, plant=None):
    """Mean of two branches over the same input; a branch passes through a full-width RMS norm first."""
    left = chunk_attention(h, sub(W, 'left.'), c['left'], eps, plant)
    right = retention(h, sub(W, 'right.'), c['right'], eps)
    return 0.5 * (rms(left, eps) * W['left.out'] + rms(right, eps) * W['right.out'])


def swiglu(h, W):
    return (silu(h @ W['gate'].T) * (h @ W['up'].T)) @ W['down'].T


def forward(cfg, W, tokens, layers_out=None, plant=None):
    """Logits [T, vocab] of a whole sequence.  cfg: the parsed config.json; W: tensor name -> array."""
    W = {n: np.asarray(a, F) for n, a in W.items()}
    groups, eps = cfg['norm']['groups'], cfg['norm']['eps']
    x = W['embed'][np.asarray(tokens)]
    for i, L in enumerate(cfg['layers']):
        p = f'l{i}.'
        h = group_norm(x, W[p + 'norm1'], groups, eps)
        mix = sub(W, p + 'mix.')
        if L['type'] == 'channel_delta':
            x = x + channel_delta(h, mix, L['mixer'], eps)
        else:
            x = x + parallel(h, mix, L['mixer'], eps, plant)
        if L['mlp'] is not None:
            x = x + swiglu(group_norm(x, W[p + 'norm2'], groups, eps), sub(W, p + 'mlp.'))
        if layers_out is not None:
            layers_out.append(x.copy())
    return group_norm(x, W['final.norm'], groups, eps) @ W['head'].T
