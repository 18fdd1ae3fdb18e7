"""Plain float64 model of the Roravik design, written from its equations: one function per mechanism, whole sequences, no cache, no
batching -- nothing here is shared with the engine.  `cfg` is the parsed config.json, `w` maps tensor names to float64 arrays.

A block has a norm ahead of each sublayer and one behind it: x += N1b(mixer(N1 x)); x += N2b(ff(N2 x)), N an RMS norm whose weight is
stored around zero.  A range of layers runs several times on the same weights; from the second pass on the stream is joined by the
embedding output where the pass begins.
Mixers: `retention` -- a state per head with one fixed decay, S <- g S + k v^T, o = S^T q, rotated queries and keys, unit-RMS
heads, a silu gate.  `parallel` -- left: windowed grouped-query attention with convolved projections, rotation, capped scores and a sink in
the soft-max denominator; right: a state per head with a decay per token and key channel, every projection reading its own mix of the
token and its predecessor, a bonus for the current token; the result is a weighted sum of both.
Feed-forwards: a clamped gated unit, or sigmoid-routed gated-silu experts chosen inside the best groups, plus a gated shared expert."""
import json
import math
import os
import struct

import numpy as np


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def rms(x, eps):
    """x divided by its root mean square over the last axis"""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def rotate_half(x, pos, dims, base):
    """x [T, ..., n]: channels (i, i + dims / 2), i < dims / 2, turn by pos * base^(-2i / dims); channels from dims on pass"""
    out = x.copy()
    if dims <= 0:
        return out
    half = dims // 2
    f = float(base) ** (-2.0 * np.arange(half, dtype=np.float64) / dims)
    ang = np.asarray(pos, np.float64).reshape((-1,) + (1,) * (x.ndim - 1)) * f
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * np.cos(ang) - v * np.sin(ang)
    out[..., half:dims] = v * np.cos(ang) + u * np.sin(ang)
    return out


def short_conv(u, w):
    """u [T, C], w [C, n] -> out[t] = w[:, n-1] u[t] + w[:, n-2] u[t-1] + ...; rows ahead of the sequence count as zero"""
    taps = w.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, u.shape[1])), u])
    return sum(w[:, j] * pad[j:j + len(u)] for j in range(taps))


def retention_recurrence(q, k, v, decay, state=None):
    """q, k [T, d], v [T, dv]: S <- decay S + k v^T; o = S^T q.  Returns (o [T, dv], S)"""
    S = np.zeros((q.shape[1], v.shape[1])) if state is None else state.copy()
    o = np.zeros((len(q), v.shape[1]))
    for t in range(len(q)):
        S = decay * S + np.outer(k[t], v[t])
        o[t] = S.T @ q[t]
    return o, S


def retention_mixer(h, m, w, p, eps):
    T, H, D, V = len(h), int(m['heads']), int(m['dim']), int(m['vdim'])
    dims, base = int(m['rot']['dims']), m['rot']['base']
    q = rotate_half((h @ w[p + 'q'].T).reshape(T, H, D), np.arange(T), dims, base)
    k = rotate_half((h @ w[p + 'k'].T).reshape(T, H, D), np.arange(T), dims, base) * D ** -0.5
    v = (h @ w[p + 'v'].T).reshape(T, H, V)
    o = np.stack([rms(retention_recurrence(q[:, a], k[:, a], v[:, a], float(m['decay'][a]))[0], eps) for a in range(H)], 1)
    return (o.reshape(T, H * V) * silu(h @ w[p + 'g'].T)) @ w[p + 'o'].T


def sink_softmax(s, visible, sink):
    """scores [T, T], visible [T, T] -> weights; the denominator also holds exp(sink)"""
    s = np.where(visible, s, -np.inf)
    top = np.maximum(s.max(-1, keepdims=True), sink)
    e = np.exp(s - top)
    return e / (e.sum(-1, keepdims=True) + np.exp(sink - top))


def window_mask(T, size):
    """row i sees column j iff 0 <= i - j < size"""
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (d >= 0) & (d < size)


def attention_mixer(h, m, w, p):
    T, H, G, D, V = len(h), int(m['heads']), int(m['kv_heads']), int(m['dim']), int(m['vdim'])
    q, k, v = (short_conv(h @ w[p + t].T, w[p + t + '.conv']) for t in 'qkv')
    dims, base = int(m['rot']['dims']), m['rot']['base']
    q = rotate_half(q.reshape(T, H, D), np.arange(T), dims, base)
    k = rotate_half(k.reshape(T, G, D), np.arange(T), dims, base)
    v = v.reshape(T, G, V)
    cap, vis = float(m['softcap']), window_mask(T, int(m['mask']['size']))
    out = np.zeros((T, H, V))
    for a in range(H):
        g = a // (H // G)
        s = cap * np.tanh(q[:, a] @ k[:, g].T * float(m['scale']) / cap)
        out[:, a] = sink_softmax(s, vis, w[p + 'sink'][a]) @ v[:, g]
    return out.reshape(T, H * V) @ w[p + 'o'].T


def previous(h):
    """the predecessor's row, zeros ahead of the first"""
    return np.concatenate([np.zeros_like(h[:1]), h[:-1]])


def bonus_recurrence(r, k, v, decay, u, state=None):
    """r, k, decay [T, d], v [T, dv], u [d]: the token reads the state of its
    predecessors plus its own pair weighted by u, o = r^T S + (r . (u k)) v; then S <- diag(decay) S + k v^T"""
    S = np.zeros((r.shape[1], v.shape[1])) if state is None else state.copy()
    o = np.zeros((len(r), v.shape[1]))
    for t in range(len(r)):
        o[t] = (S + np.outer(u * k[t], v[t])).T @ r[t]
        S = decay[t][:, None] * S + np.outer(k[t], v[t])
    return o, S


def channel_decay(x, w, p):
    """exp(-exp(w2 tanh(w1 x) + w0)) per key channel"""
    return np.exp(-np.exp(np.tanh(x @ w[p + 'w1'].T) @ w[p + 'w2'].T + w[p + 'w0']))


def time_mixer(h, m, w, p, eps):
    T, H, D = len(h), int(m['heads']), int(m['dim'])
    mix = {s: h + (previous(h) - h) * w[p + 'mu.' + s] for s in 'rkvgw'}
    r, k, v = ((mix[s] @ w[p + s].T).reshape(T, H, D) for s in 'rkv')
    gate = silu(mix['g'] @ w[p + 'g'].T)
    dec = channel_decay(mix['w'], w, p).reshape(T, H, D)
    o = np.stack([rms(bonus_recurrence(r[:, a], k[:, a], v[:, a], dec[:, a], w[p + 'u'][a])[0], eps) for a in range(H)], 1)
    return (o.reshape(T, H * D) * w[p + 'norm'] * gate) @ w[p + 'o'].T


def parallel_mixer(h, m, w, p, eps):
    return (float(m['left_scale']) * attention_mixer(h, m['left'], w, p + 'left.')
            + float(m['right_scale']) * time_mixer(h, m['right'], w, p + 'right.', eps))


def clamped_ff(h, w, p, limit):
    g = np.minimum(h @ w[p + 'gate'].T, limit)
    u = np.clip(h @ w[p + 'up'].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + 'down'].T


def gated_silu_ff(h, w, p):
    return (silu(h @ w[p + 'gate'].T) * (h @ w[p + 'up'].T)) @ w[p + 'down'].T


def route(z, correction, r):
    """router logits [T, E] -> weights [T, E], zero where an expert is not chosen"""
    T, E = z.shape
    count, keep, top = int(r['groups']['count']), int(r['groups']['keep']), int(r['top'])
    s = sigmoid(z)
    choice = s + correction
    per = E // count
    gs = np.sort(choice.reshape(T, count, per), -1)[..., -2:].sum(-1)
    out = np.zeros((T, E))
    for t in range(T):
        kept = np.argsort(-gs[t], kind='stable')[:keep]
        c = np.full(E, -np.inf)
        for g in kept:
            c[g * per:(g + 1) * per] = choice[t, g * per:(g + 1) * per]
        ids = np.argsort(-c, kind='stable')[:top]
        out[t, ids] = s[t, ids] / (s[t, ids].sum() + 1e-20)
    return out


def router_gap(z, correction, r):
    """how close the closest of a token's choices is, [T]: between the last kept and the first dropped group, and between the last chosen and
    the first refused expert of the kept groups"""
    T, E = z.shape
    count, keep, top = int(r['groups']['count']), int(r['groups']['keep']), int(r['top'])
    per, gap = E // count, np.full(T, np.inf)
    choice = sigmoid(z) + correction
    gs = np.sort(choice.reshape(T, count, per), -1)[..., -2:].sum(-1)
    for t in range(T):
        order = np.argsort(-gs[t], kind='stable')
        if keep < count:
            gap[t] = gs[t, order[keep - 1]] - gs[t, order[keep]]
        c = np.sort(np.concatenate([choice[t, g * per:(g + 1) * per] for g in order[:keep]]))[::-1]
        if top < len(c):
            gap[t] = min(gap[t], c[top - 1] - c[top])
    return gap


def expert_ff(h, m, w, p):
    wt = route(h @ w[p + 'router'].T, w[p + 'correction'], m['router'])
    y = sum(wt[:, e:e + 1] * gated_silu_ff(h, w, p + f'e{e}.') for e in range(wt.shape[1]))
    return y + sigmoid(h @ w[p + 'shared.sg'].T) * gated_silu_ff(h, w, p + 'shared.')


def layer_runs(cfg):
    """[(layer, opens a later pass of the loop)] in the order they run"""
    n, lp = len(cfg['layers']), cfg.get('loop') or {}
    start, stop, times = int(lp.get('start', 0)), int(lp.get('stop', 0)), int(lp.get('times', 1))
    if stop <= start:
        return [(i, False) for i in range(n)]
    runs = [(i, False) for i in range(start)]
    for t in range(times):
        runs += [(i, t > 0 and i == start) for i in range(start, stop)]
    return runs + [(i, False) for i in range(stop, n)]


def block(x, i, L, w, eps, taps=None):
    p = f'l{i}.'
    h = norm(x, w[p + 'norm1'], eps)
    if L['type'] == 'retention':
        y = retention_mixer(h, L['mixer'], w, p + 'mix.', eps)
    elif L['type'] == 'parallel':
        y = parallel_mixer(h, L['mixer'], w, p + 'mix.', eps)
    else:
        raise NotImplementedError(L['type'])
    x = x + norm(y, w[p + 'norm1b'], eps)
    m = L.get('mlp')
    if m is not None:
        h = norm(x, w[p + 'norm2'], eps)
        if m['kind'] == 'moe' and taps is not None:
            taps.append(router_gap(h @ w[p + 'mlp.router'].T, w[p + 'mlp.correction'], m['router']))
        y = clamped_ff(h, w, p + 'mlp.', float(m['limit'])) if m['kind'] == 'dense' else expert_ff(h, m, w, p + 'mlp.')
        x = x + norm(y, w[p + 'norm2b'], eps)
    return x


def forward(cfg, w, tokens, return_layers=False, taps=None):
    """logits [T, vocab] of one sequence (and the stream behind every layer run); `taps` collects router_gap() of every expert layer run"""
    eps = float(cfg['norm']['eps'])
    x0 = w['embed'][np.asarray(tokens)] * float(cfg['embedding']['scale'])
    x, trail = x0, []
    for i, again in layer_runs(cfg):
        x = block(x + x0 if again else x, i, cfg['layers'][i], w, eps, taps)
        trail.append(x)
    logits = norm(x, w['final.norm'], eps) @ w['embed'].T
    cap = float(cfg['logit_softcap'])
    logits = cap * np.tanh(logits / cap)
    return (logits, np.stack(trail)) if return_layers else logits


# ---- configurations, random weights, checkpoints ------------------------------------------------------------------------------------
def retention_layer(heads, dim, vdim, decay, base=10000.0, rot_dims=None, mlp=None):
    return {'type': 'retention', 'mixer': {'heads': heads, 'dim': dim, 'vdim': vdim, 'decay': list(decay),
                                           'rot': {'base': base, 'dims': dim if rot_dims is None else rot_dims}}, 'mlp': mlp}


def parallel_layer(heads, kv_heads, dim, vdim, window, r_heads, r_dim, scale=None, softcap=20.0, conv=3, base=10000.0, rot_dims=None,
                   left_scale=0.7, right_scale=1.2, mlp=None):
    left = {'heads': heads, 'kv_heads': kv_heads, 'dim': dim, 'vdim': vdim, 'conv': conv, 'scale': dim ** -0.5 if scale is None else scale,
            'softcap': softcap, 'mask': {'size': window}, 'rot': {'base': base, 'dims': dim if rot_dims is None else rot_dims}}
    return {'type': 'parallel', 'mixer': {'left': left, 'right': {'heads': r_heads, 'dim': r_dim}, 'left_scale': left_scale,
                                          'right_scale': right_scale}, 'mlp': mlp}


def dense(ff, limit=1.5):
    return {'kind': 'dense', 'ff': ff, 'limit': limit}


def moe(experts, top, ff, groups, keep, shared):
    return {'kind': 'moe', 'expert': {'ff': ff}, 'router': {'experts': experts, 'top': top, 'groups': {'count': groups, 'keep': keep}},
            'shared': {'ff': shared}}


def make_config(width, vocab, layers, eps=1e-5, embed_scale=1.5, logit_softcap=12.0, loop=None):
    cfg = {'architecture': 'Roravik', 'width': width, 'vocab': vocab, 'norm': {'eps': eps}, 'embedding': {'scale': embed_scale},
           'logit_softcap': logit_softcap, 'layers': layers}
    if loop:
        cfg['loop'] = {'start': loop[0], 'stop': loop[1], 'times': loop[2]}
    return cfg


def tensor_shapes(cfg, decay_rank=6):
    """decay_rank: the inner size of the decay's two-matrix projection (the tensors' own)"""
    W, V = int(cfg['width']), int(cfg['vocab'])
    out = {'embed': (V, W), 'final.norm': (W,)}
    for i, L in enumerate(cfg['layers']):
        p, m, f = f'l{i}.', L['mixer'], L.get('mlp')
        for n in ('norm1', 'norm1b') + (('norm2', 'norm2b') if f is not None else ()):
            out[p + n] = (W,)
        if L['type'] == 'retention':
            H, D, Vd = m['heads'], m['dim'], m['vdim']
            for t, n in (('q', H * D), ('k', H * D), ('v', H * Vd), ('g', H * Vd)):
                out[p + 'mix.' + t] = (n, W)
            out[p + 'mix.o'] = (W, H * Vd)
        else:
            a, b, l, r = m['left'], m['right'], p + 'mix.left.', p + 'mix.right.'
            H, G, D, Vd, taps = a['heads'], a['kv_heads'], a['dim'], a['vdim'], a['conv']
            for t, n in (('q', H * D), ('k', G * D), ('v', G * Vd)):
                out[l + t], out[l + t + '.conv'] = (n, W), (n, taps)
            out[l + 'sink'], out[l + 'o'] = (H,), (W, H * Vd)
            n = b['heads'] * b['dim']
            for t in 'rkvgw':
                out[r + 'mu.' + t] = (W,)
            for t in 'rkvg':
                out[r + t] = (n, W)
            out.update({r + 'w1': (decay_rank, W), r + 'w2': (n, decay_rank), r + 'w0': (n,), r + 'u': (b['heads'], b['dim']), r + 'norm': (n,),
                        r + 'o': (W, n)})
        if f is None:
            continue
        if f['kind'] == 'dense':
            out.update({p + 'mlp.gate': (f['ff'], W), p + 'mlp.up': (f['ff'], W), p + 'mlp.down': (W, f['ff'])})
        else:
            E = f['router']['experts']
            out.update({p + 'mlp.router': (E, W), p + 'mlp.correction': (E,), p + 'mlp.shared.sg': (1, W)})
            for e, ff in [(f'e{e}', f['expert']['ff']) for e in range(E)] + [('shared', f['shared']['ff'])]:
                q = p + f'mlp.{e}.'
                out.update({q + 'gate': (ff, W), q + 'up': (ff, W), q + 'down': (W, ff)})
    return out


def bf16_round(x):
    b = np.asarray(x, np.float32).view(np.uint32).astype(np.uint64)
    b = ((b + 0x7FFF + ((b >> 16) & 1)) >> 16) << 16
    return b.astype(np.uint32).view(np.float32).astype(np.float64)


def random_weights(cfg, seed=0, decay_rank=6):
    """bf16-representable float64 weights: matrices N(0, 1 / inputs), zero-centred norm weights, the decays' offsets spread over states that
    forget at once and states that hold for hundreds of tokens, mixes over 0 .. 1, corrections that move the experts' order"""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in tensor_shapes(cfg, decay_rank).items():
        leaf = name.split('.')[-1]
        if name == 'embed':
            a = rng.standard_normal(shape) / math.sqrt(shape[-1]) * 3.0
        elif leaf in ('norm1', 'norm1b', 'norm2', 'norm2b') or name == 'final.norm':
            a = 0.15 * rng.standard_normal(shape)
        elif leaf == 'norm':
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif '.mu.' in name:
            a = rng.uniform(0.0, 1.0, shape)
        elif leaf == 'w0':
            a = rng.uniform(-6.0, 1.0, shape)
        elif leaf == 'conv':
            a = rng.standard_normal(shape) / math.sqrt(shape[-1])
        elif leaf in ('sink', 'u'):
            a = rng.standard_normal(shape)
        elif leaf == 'correction':
            a = 0.3 * rng.standard_normal(shape)
        else:
            a = rng.standard_normal(shape) / math.sqrt(shape[-1])
        w[name] = bf16_round(a)
    return w


def bf16_bits(x):
    b = np.asarray(x, np.float32).view(np.uint32)
    return (b >> 16).astype(np.uint16)


def write_checkpoint(folder, cfg, w):
    """config.json + model.safetensors (bf16) in `folder`"""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, 'config.json'), 'w') as f:
        json.dump(cfg, f)
    header, blobs, off = {}, [], 0
    for name, a in w.items():
        raw = bf16_bits(a).tobytes()
        header[name] = {'dtype': 'BF16', 'shape': list(np.shape(a)), 'data_offsets': [off, off + len(raw)]}
        blobs.append(raw)
        off += len(raw)
    hj = json.dumps(header).encode()
    hj += b' ' * (-len(hj) % 8)
    with open(os.path.join(folder, 'model.safetensors'), 'wb') as f:
        f.write(struct.pack('<Q', len(hj)) + hj + b''.join(blobs))
