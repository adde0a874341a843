"""Plain float32 restatement of the Lugasun decoder, one function per mechanism, for the tests (CPU, eager, slow).

No caches, no batching, no fusion: every function takes whole sequences [tokens, features] and follows the equation in its
docstring.  `forward` strings them together and can return the residual stream after every layer pass.  Weights come as a dict of
tensors under the checkpoint's names; the configuration is the parsed config.json.
"""
import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * w


def rotate(x, base, dims, start=0):
    """x [tokens, heads, dim]: entries i and i + dims / 2 of a head turn by p * base^(-2 i / dims); entries from `dims` on stay."""
    if not dims:
        return x
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64).float()
    a = torch.arange(start, start + x.shape[0]).float()[:, None] * f
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat([u * c - v * s, v * c + u * s, rest], -1)


def soft_cap(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def visible(n, size):
    """[query, key]: keys up to the query that lie in the query's chunk of `size` positions (None: all keys up to the query)."""
    i = torch.arange(n)
    seen = i[None, :] <= i[:, None]
    return seen & (i[None, :] // size == i[:, None] // size) if size else seen


def grouped_attention(q, k, v, scale, cap, size):
    """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]: softmax(cap tanh(scale q k / cap)) v over the visible keys; H / G neighbouring query heads share a key head."""
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    seen = visible(n, size)
    out = []
    for h in range(H):
        g = h // (H // G)
        s = soft_cap(q[:, h] @ k[:, g].T * scale, cap).masked_fill(~seen, -math.inf)
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out.append((e / e.sum(-1, keepdim=True)) @ v[:, g])
    return torch.stack(out, 1)


def attention(w, p, mix, h, eps):
    """Normed, rotated queries and keys; chunked, soft-capped softmax attention; output projection."""
    n, H, G, d, dv = h.shape[0], mix['heads'], mix['kv_heads'], mix['dim'], mix['vdim']
    q = norm((h @ w[p + 'q'].float().T).view(n, H, d), w[p + 'q.norm'].float(), eps)
    k = norm((h @ w[p + 'k'].float().T).view(n, G, d), w[p + 'k.norm'].float(), eps)
    v = (h @ w[p + 'v'].float().T).view(n, G, dv)
    rot = mix.get('rot') or {'base': 1.0, 'dims': 0}
    q, k = rotate(q, rot['base'], rot['dims']), rotate(k, rot['base'], rot['dims'])
    o = grouped_attention(q, k, v, mix['scale'], mix.get('softcap'), (mix.get('mask') or {}).get('size'))
    return o.reshape(n, H * dv) @ w[p + 'o'].float().T


def decayed_recurrence(q, k, v, decay):
    """S <- decay S + k_t v_t^T, o_t = S^T q_t for one head, token by token from S = 0; q, k [n, d], v [n, dv]."""
    S, out = torch.zeros(k.shape[1], v.shape[1]), []
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        out.append(S.T @ q[t])
    return torch.stack(out)


def retention(w, p, mix, h, eps):
    """Rotated queries and keys (keys over sqrt(dim)), a decayed recurrence per head, rows of a head over their root mean square, gated by silu(W_g h), output projection."""
    n, H, d, dv = h.shape[0], mix['heads'], mix['dim'], mix['vdim']
    rot = mix.get('rot') or {'base': 1.0, 'dims': 0}
    q = rotate((h @ w[p + 'q'].float().T).view(n, H, d), rot['base'], rot['dims'])
    k = rotate((h @ w[p + 'k'].float().T).view(n, H, d), rot['base'], rot['dims']) * d ** -0.5
    v = (h @ w[p + 'v'].float().T).view(n, H, dv)
    o = torch.stack([rms(decayed_recurrence(q[:, i], k[:, i], v[:, i], mix['decay'][i]), eps) for i in range(H)], 1)
    g = h @ w[p + 'g'].float().T
    return (o.reshape(n, H * dv) * (g * torch.sigmoid(g))) @ w[p + 'o'].float().T


def side_by_side(w, p, mix, h, eps):
    return mix['left_scale'] * attention(w, p + 'left.', mix['left'], h, eps) + mix['right_scale'] * retention(w, p + 'right.', mix['right'], h, eps)


def feed_forward(w, p, h):
    """W_down relu(W_up h)^2"""
    return torch.relu(h @ w[p + 'up'].float().T).square() @ w[p + 'down'].float().T


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def token_side(w, i, dim, x, tokens, eps):
    """What layer i adds for its tokens: rms(W_proj (gelu(W_gate x) * e)) * weight with e = the layer's part of the token's row in the side table."""
    p = f'l{i}.side.'
    e = w['side.embed'].float()[tokens][:, i * dim:(i + 1) * dim]
    return norm((gelu_tanh(x @ w[p + 'gate'].float().T) * e) @ w[p + 'proj'].float().T, w[p + 'norm'].float(), eps)


def layer(w, cfg, i, x, tokens):
    p, spec, eps = f'l{i}.', cfg['layers'][i], cfg['norm']['eps']
    x = x + side_by_side(w, p + 'mix.', spec['mixer'], norm(x, w[p + 'norm1'].float(), eps), eps)
    if spec.get('mlp') is not None:
        x = x + feed_forward(w, p + 'mlp.', norm(x, w[p + 'norm2'].float(), eps))
    if cfg.get('token_side'):
        x = x + token_side(w, i, cfg['token_side']['dim'], x, tokens, eps)
    return x


def mix_in(w, x, x0):
    """Ahead of every pass of the looped span: W_in [x; x0], x0 the embedding."""
    return torch.cat([x, x0], -1) @ w['loop.in'].float().T


def passes(cfg):
    """(layer index, does a pass of the looped span start here) of every layer pass."""
    n, lp = len(cfg['layers']), cfg.get('loop')
    if not lp:
        return [(i, False) for i in range(n)]
    span = [(i, i == lp['start']) for i in range(lp['start'], lp['stop'])]
    return [(i, False) for i in range(lp['start'])] + span * lp['times'] + [(i, False) for i in range(lp['stop'], n)]


def forward(w, cfg, tokens, with_layers=False):
    """tokens [n] -> logits [n, vocab] (and the residual stream after every layer pass)."""
    tokens = torch.as_tensor(tokens)
    x0 = w['embed'].float()[tokens]
    x, xs = x0, []
    for i, starts in passes(cfg):
        if starts:
            x = mix_in(w, x, x0)
        x = layer(w, cfg, i, x, tokens)
        xs.append(x)
    z = norm(x, w['final.norm'].float(), cfg['norm']['eps']) @ w['embed'].float().T
    return (z, xs) if with_layers else z


def greedy(w, cfg, prompt, n_new, eos=None):
    """Greedy continuation by whole forwards; -> (ids, top-2 margin of every pick)."""
    ids, out, margins = list(prompt), [], []
    for _ in range(n_new):
        z = forward(w, cfg, ids)[-1]
        t = z.topk(2).values
        out.append(int(z.argmax()))
        margins.append(float(t[0] - t[1]))
        ids.append(out[-1])
        if eos is not None and out[-1] == eos:
            break
    return out, margins
