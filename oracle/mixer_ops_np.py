"""NumPy statement of the layered-mixer ops of the surface (include/adamah_hip.h), on the oracle's flat maps.

Test infrastructure.  Token by token in float64 from the state the maps hold; results rounded to float32 when stored
(bfloat16 maps: to bfloat16).  No counterpart in the reference, so what pins these ops is `mixers_np.py`, which states
the mechanisms over whole sequences and never touches a map.
"""
import numpy as np

F = np.float64
_LINEAR = ("w n k k_stride src src_stride groups eps wt wt_len gate gate_stride gate_act opnd ready out out_stride epi "
           "out_opnd out_opnd_stride wt_add bias biased branch branch_stride branch_wt branched res_out res_stride keep keep_stride "
           "kept tail tail_out tail_stride")
_MERGE = "a b stride wa wb dst dst_stride dim eps scale store"
_DELTA = ("heads kv_heads dim vdim taps x x_stride x_b cq ck cv a_log dt_bias out out_stride state_map s_off conv_off "
          "seq_stride")
_RET = "heads dim vdim rot_dims freq decay x x_stride x_q x_k x_v out out_stride state_map s_off seq_stride"
_ATT = ("heads kv_heads dim vdim chunk x x_stride x_q x_k x_v r1 r2 scale eps out out_stride cache_map k_off v_off "
        "seq_stride")
_WIN = ("heads kv_heads dim vdim window x x_stride x_q x_k x_v slope sink has_sink qk_norm scale eps softcap temp_coef temp_every "
        "out out_stride cache_map k_off v_off seq_stride")
_SSM = ("heads groups state vdim taps x x_stride x_c x_dt conv conv_b dt_bias a_log skip out out_stride state_map s_off conv_off "
        "seq_stride")
_MOE = ("experts identity top ff ff_stride width k_stride gate_up gate_up_step down down_step logits logits_stride correction x "
        "x_stride opnd act act_opnd shared_ff shared_ff_stride shared_down shared_act out out_stride epi")
_BIGRAM = "table vocab width dst scale pairs buckets mul_prev mul_cur state_map prev_off seq_stride"
_FLOATS = {"eps", "scale", "wt_add", "softcap", "temp_coef"}


class _S:
    pass


def _silu(z):
    return z / (1.0 + np.exp(-z))


def _sig(z):
    return 1.0 / (1.0 + np.exp(-z))


class MixerOps:
    def _spec(self, h, names):
        w = self.res[h].view(np.uint32)
        s = _S()
        for i, n in enumerate(names.split()):
            setattr(s, n, float(w[i:i + 1].view(np.float32)[0]) if n in _FLOATS else int(w[i]))
        return s

    def _get(self, mid, off, n):
        d = self.maps[mid].data[off:off + n]
        assert d.size == n, "range outside the map"
        return (d.astype(np.uint32) << 16).view(np.float32).astype(F) if d.dtype == np.uint16 else d.astype(F)

    def _put(self, mid, off, v):
        v = np.ascontiguousarray(v, np.float32).reshape(-1)
        d = self.maps[mid].data
        assert off + v.size <= d.size, "range outside the map"
        if d.dtype == np.uint16:
            u = v.view(np.uint32)
            v = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)
        d[off:off + v.size] = v

    def embed_tokens_dev(self, map_act, map_src, locs, src_row0, dst, m, E, V, scale=1.0):
        toks = self._get(map_act, 0, self.maps[map_act].n)[self.res[locs].view(np.uint32)[:m]]
        for r, t in enumerate(toks):
            ok = 0 <= t < V
            self._put(map_act, dst + r * E, self._get(map_src, src_row0 + int(t) * E, E) * scale if ok else np.zeros(E))

    def linear_dev(self, map_act, map_opnd, map_wt, h, h_rows, rows):
        s = self._spec(h, _LINEAR)
        idx = self.res[h_rows].view(np.uint32)[:rows] if h_rows else range(rows)
        W = self._get(map_wt, s.w, s.n * s.k_stride).reshape(s.n, s.k_stride)
        assert not np.any(W[:, s.k:]), "columns beyond k must be zero"
        for r, i in enumerate(idx):
            i = int(i)
            if rows > 1 and s.ready:
                x = self._get(map_opnd, s.opnd + r * s.k_stride, s.k)
            else:
                x = self._get(map_act, s.src + i * s.src_stride, s.k)
                if s.branched:
                    b = self._get(map_act, s.branch + i * s.branch_stride, s.k)
                    x = x + b / np.sqrt(np.mean(b * b) + s.eps) * (s.wt_add + self._get(map_act, s.branch_wt, s.k))
                    if s.branched == 2:
                        self._put(map_act, s.res_out + i * s.res_stride, x)
                if s.groups:
                    if s.gate_act == 3:
                        x = x * _silu(self._get(map_act, s.gate + i * s.gate_stride, s.k))
                    y = x.reshape(s.groups, -1)
                    x = (y / np.sqrt(np.mean(y * y, axis=1, keepdims=True) + s.eps)).reshape(-1)
                    if s.wt_len:
                        x = x * np.resize(s.wt_add + self._get(map_act, s.wt, s.wt_len), s.k)
                    if s.gate_act in (1, 2):
                        x = x * (_sig, _silu)[s.gate_act - 1](self._get(map_act, s.gate + i * s.gate_stride, s.k))
                if s.kept:
                    self._put(map_act, s.keep + i * s.keep_stride, x)
                if rows > 1:
                    self._put(map_opnd, s.opnd + r * s.k_stride, x)
                    x = self._get(map_opnd, s.opnd + r * s.k_stride, s.k)
            y = W[:, :s.k] @ x
            if s.biased:
                y = y + self._get(map_act, s.bias, s.n)
            if s.epi == 2:
                if s.tail:
                    self._put(map_act, s.tail_out + r * s.tail_stride, y[s.n - s.tail:])
                y = y[:s.n - s.tail].reshape(-1, 2, 16)
                y = (_silu(y[:, 0]) * y[:, 1]).reshape(-1)
                if rows > 1:
                    self._put(map_opnd, s.out_opnd + r * s.out_opnd_stride, y)
                    continue
            o = s.out + r * s.out_stride
            self._put(map_act, o, y + self._get(map_act, o, y.size) if s.epi == 1 else y)

    def linear_argmax_dev(self, map_act, map_opnd, map_wt, h, h_dst, rows):
        self.linear_dev(map_act, map_opnd, map_wt, h, 0, rows)
        s = self._spec(h, _LINEAR)
        for r, d in enumerate(self.res[h_dst].view(np.uint32)[:rows]):
            self._put(map_act, int(d), [np.argmax(self._get(map_act, s.out + r * s.out_stride, s.n))])

    def merge_norm_dev(self, map_act, h, rows):
        s = self._spec(h, _MERGE)
        for r in range(rows):
            y = 0.0
            for src, w in ((s.a, s.wa), (s.b, s.wb)):
                x = self._get(map_act, src + r * s.stride, s.dim)
                y = y + x / np.sqrt(np.mean(x * x) + s.eps) * self._get(map_act, w, s.dim)
            d = s.dst + r * s.dst_stride
            self._put(map_act, d, (0.0 if s.store else self._get(map_act, d, s.dim)) + s.scale * y)

    @staticmethod
    def _tokens(n_seq, rows, seq0, pos):
        """(row, slot, position) of every token of a call."""
        assert n_seq == 1 or rows == 1
        return [(r, seq0, pos + r) for r in range(rows)] if n_seq == 1 else [(i, seq0 + i, pos) for i in range(n_seq)]

    def delta_rule_dev(self, map_act, map_opnd, map_wt, h, h_dec, h_gate, n_seq, rows, seq0, pos):
        s = self._spec(h, _DELTA)
        H, KH, D, V, J = s.heads, s.kv_heads, s.dim, s.vdim, s.taps
        n_ch = 2 * KH * D + H * V
        conv = np.concatenate([self._get(map_act, o, n * J).reshape(n, J) for o, n in ((s.cq, KH * D), (s.ck, KH * D), (s.cv, H * V))])
        pick = np.arange(H) // (H // KH)
        n_tok = n_seq * rows
        dec, gate = self._spec(h_dec, _LINEAR), self._spec(h_gate, _LINEAR)
        self.linear_dev(map_act, map_opnd, map_wt, h_dec, 0, n_tok)
        self.linear_dev(map_act, map_opnd, map_wt, h_gate, 0, n_tok)
        for r, slot, p in self._tokens(n_seq, rows, seq0, pos):
            base = slot * s.seq_stride
            x = self._get(map_act, s.x + r * s.x_stride, s.x_stride)
            ring = self._get(s.state_map, base + s.conv_off, J * n_ch).reshape(J, n_ch)
            ring[p % J] = x[:n_ch]
            self._put(s.state_map, base + s.conv_off, ring)
            z = sum(conv[:, J - 1 - j] * ring[(p - j) % J] for j in range(J) if j <= p)
            z = _silu(z)
            un = lambda a: a / np.sqrt(np.sum(a * a, axis=-1, keepdims=True) + 1e-6)
            q = (un(z[:KH * D].reshape(KH, D)) * D ** -0.5)[pick]
            k = un(z[KH * D:2 * KH * D].reshape(KH, D))[pick]
            v = z[2 * KH * D:].reshape(H, V)
            a = self._get(map_act, dec.out + r * dec.out_stride, H * D) + self._get(map_act, s.dt_bias, H * D)
            g = np.exp(-np.exp(self._get(map_act, s.a_log, H))[:, None] * np.logaddexp(0, a).reshape(H, D))
            S = self._get(s.state_map, base + s.s_off, H * D * V).reshape(H, D, V) if p else np.zeros((H, D, V))
            S = g[:, :, None] * S
            u = _sig(x[s.x_b:s.x_b + H])[:, None] * (v - np.einsum('hdv,hd->hv', S, k))
            S = S + k[:, :, None] * u[:, None, :]
            self._put(s.state_map, base + s.s_off, S)
            self._put(map_act, s.out + r * s.out_stride, np.einsum('hdv,hd->hv', S, q))

    def retention_dev(self, map_act, h, n_seq, rows, seq0, pos):
        s = self._spec(h, _RET)
        H, D, V, half = s.heads, s.dim, s.vdim, s.rot_dims // 2
        freq, dec = self._get(map_act, s.freq, half), self._get(map_act, s.decay, H)

        def rot(x, p):
            c, n = np.cos(p * freq), np.sin(p * freq)
            a, b = x[:, :half], x[:, half:2 * half]
            return np.concatenate([a * c - b * n, b * c + a * n, x[:, 2 * half:]], axis=1)
        for r, slot, p in self._tokens(n_seq, rows, seq0, pos):
            base = slot * s.seq_stride
            x = self._get(map_act, s.x + r * s.x_stride, s.x_stride)
            q = rot(x[s.x_q:s.x_q + H * D].reshape(H, D), p)
            k = rot(x[s.x_k:s.x_k + H * D].reshape(H, D), p) * D ** -0.5
            v = x[s.x_v:s.x_v + H * V].reshape(H, V)
            S = self._get(s.state_map, base + s.s_off, H * D * V).reshape(H, D, V) if p else np.zeros((H, D, V))
            S = dec[:, None, None] * S + k[:, :, None] * v[:, None, :]
            self._put(s.state_map, base + s.s_off, S)
            self._put(map_act, s.out + r * s.out_stride, np.einsum('hdv,hd->hv', S, q))

    def chunk_attention_dev(self, map_act, h, n_seq, rows, seq0, pos):
        s = self._spec(h, _ATT)
        H, G, D, V, C = s.heads, s.kv_heads, s.dim, s.vdim, s.chunk
        D8, V8 = (D + 7) // 8 * 8, (V + 7) // 8 * 8
        r1, r2 = self._get(map_act, s.r1, H), self._get(map_act, s.r2, H)
        for r, slot, p in self._tokens(n_seq, rows, seq0, pos):
            base = slot * s.seq_stride
            x = self._get(map_act, s.x + r * s.x_stride, s.x_stride)
            n = p % C + 1
            v = x[s.x_v:s.x_v + G * V].reshape(G, V)
            v = v / np.sqrt(np.mean(v * v, axis=1, keepdims=True) + s.eps)
            for g in range(G):
                k8, v8 = np.zeros(D8), np.zeros(V8)
                k8[:D], v8[:V] = x[s.x_k + g * D:s.x_k + (g + 1) * D], v[g]
                self._put(s.cache_map, base + s.k_off + (g * C + n - 1) * D8, k8)
                self._put(s.cache_map, base + s.v_off + (g * C + n - 1) * V8, v8)
            for hd in range(H):
                g = hd // (H // G)
                K = self._get(s.cache_map, base + s.k_off + g * C * D8, n * D8).reshape(n, D8)[:, :D]
                Vc = self._get(s.cache_map, base + s.v_off + g * C * V8, n * V8).reshape(n, V8)[:, :V]
                sc = (K @ x[s.x_q + hd * D:s.x_q + (hd + 1) * D]) * s.scale - r1[hd] * np.log1p(r2[hd] * np.arange(n - 1, -1, -1))
                w = np.exp(sc - sc.max())
                self._put(map_act, s.out + r * s.out_stride + hd * V, (w / w.sum()) @ Vc)

    def window_attention_dev(self, map_act, h, n_seq, rows, seq0, pos):
        s = self._spec(h, _WIN)
        H, G, D, V, R = s.heads, s.kv_heads, s.dim, s.vdim, s.window
        D8, V8 = (D + 7) // 8 * 8, (V + 7) // 8 * 8
        slope = self._get(map_act, s.slope, H)
        rms = lambda a: a / np.sqrt(np.mean(a * a, axis=-1, keepdims=True) + s.eps) if s.qk_norm else a
        for r, slot, p in self._tokens(n_seq, rows, seq0, pos):
            base = slot * s.seq_stride
            x = self._get(map_act, s.x + r * s.x_stride, s.x_stride)
            k = rms(x[s.x_k:s.x_k + G * D].reshape(G, D))
            q = rms(x[s.x_q:s.x_q + H * D].reshape(H, D))
            if s.temp_coef:
                q = q * (1.0 + s.temp_coef * np.log((p + 1) // s.temp_every + 1))
            seen = np.arange(max(0, p - R + 1), p + 1)
            for g in range(G):
                k8, v8 = np.zeros(D8), np.zeros(V8)
                k8[:D], v8[:V] = k[g], x[s.x_v + g * V:s.x_v + (g + 1) * V]
                self._put(s.cache_map, base + s.k_off + (g * R + p % R) * D8, k8)
                self._put(s.cache_map, base + s.v_off + (g * R + p % R) * V8, v8)
            for hd in range(H):
                g = hd // (H // G)
                K = self._get(s.cache_map, base + s.k_off + g * R * D8, R * D8).reshape(R, D8)[seen % R, :D]
                Vc = self._get(s.cache_map, base + s.v_off + g * R * V8, R * V8).reshape(R, V8)[seen % R, :V]
                sc = (K @ q[hd]) * s.scale
                if s.softcap:
                    sc = s.softcap * np.tanh(sc / s.softcap)
                sc = sc - slope[hd] * (p - seen)
                sink = self._get(map_act, s.sink + hd, 1)[0] if s.has_sink else -np.inf
                top = max(sc.max(), sink)
                w = np.exp(sc - top)
                self._put(map_act, s.out + r * s.out_stride + hd * V, (w / (w.sum() + np.exp(sink - top))) @ Vc)

    def state_space_dev(self, map_act, h, n_seq, rows, seq0, pos):
        s = self._spec(h, _SSM)
        H, G, N, V, J = s.heads, s.groups, s.state, s.vdim, s.taps
        n_ch = H * V + 2 * G * N
        w, b = self._get(map_act, s.conv, n_ch * J).reshape(n_ch, J), self._get(map_act, s.conv_b, n_ch)
        pick = np.arange(H) // (H // G)
        for r, slot, p in self._tokens(n_seq, rows, seq0, pos):
            base = slot * s.seq_stride
            x = self._get(map_act, s.x + r * s.x_stride, s.x_stride)
            ring = self._get(s.state_map, base + s.conv_off, J * n_ch).reshape(J, n_ch)
            ring[p % J] = x[s.x_c:s.x_c + n_ch]
            self._put(s.state_map, base + s.conv_off, ring)
            z = _silu(b + sum(w[:, J - 1 - j] * ring[(p - j) % J] for j in range(J) if j <= p))
            u = z[:H * V].reshape(H, V)
            B, C = (z[H * V + i * G * N:H * V + (i + 1) * G * N].reshape(G, N)[pick] for i in (0, 1))
            dt = np.logaddexp(0, x[s.x_dt:s.x_dt + H] + self._get(map_act, s.dt_bias, H))
            g = np.exp(-np.exp(self._get(map_act, s.a_log, H)) * dt)
            S = self._get(s.state_map, base + s.s_off, H * N * V).reshape(H, N, V) if p else np.zeros((H, N, V))
            S = g[:, None, None] * S + dt[:, None, None] * B[:, :, None] * u[:, None, :]
            self._put(s.state_map, base + s.s_off, S)
            self._put(map_act, s.out + r * s.out_stride, np.einsum('hnv,hn->hv', S, C) + self._get(map_act, s.skip, H)[:, None] * u)

    def experts_dev(self, map_act, map_opnd, map_wt, h, h_shared, rows):
        s = self._spec(h, _MOE)
        n, E = s.experts + s.identity, s.width
        if s.shared_ff and rows > 1:
            sh = self._spec(h_shared, _LINEAR)
            self.linear_dev(map_act, map_opnd, map_wt, h_shared, 0, rows)
        F16 = (s.ff + 15) // 16 * 16
        for r in range(rows):
            z = self._get(map_act, s.logits + r * s.logits_stride, n + (1 if s.shared_ff else 0))
            sc = np.exp(z[:n] - z[:n].max())
            sc = sc / sc.sum()
            ids = np.argsort(-(sc + self._get(map_act, s.correction, n)), kind='stable')[:s.top]
            h32 = self._get(map_act, s.x + r * s.x_stride, E)
            x = self._get(map_opnd, s.opnd + r * s.k_stride, E) if rows > 1 else h32
            y = np.zeros(E)
            for j, e in enumerate(int(i) for i in ids):
                if e >= s.experts:
                    y += sc[e] * h32
                    continue
                gu = (self._get(map_wt, s.gate_up + e * s.gate_up_step, 2 * F16 * s.k_stride).reshape(-1, s.k_stride)[:, :E] @ x).reshape(-1, 2, 16)
                a = (_silu(gu[:, 0]) * gu[:, 1]).reshape(-1)[:s.ff]
                if rows > 1:
                    o = s.act_opnd + (r * s.top + j) * s.ff_stride
                    self._put(map_opnd, o, a)
                    a = self._get(map_opnd, o, s.ff)
                y += sc[e] * (self._get(map_wt, s.down + e * s.down_step, E * s.ff_stride).reshape(E, s.ff_stride)[:, :s.ff] @ a)
            if s.shared_ff:
                if rows > 1:
                    v = self._get(map_act, sh.out + r * sh.out_stride, E)
                else:
                    W = self._get(map_wt, s.shared_down, E * s.shared_ff_stride).reshape(E, s.shared_ff_stride)[:, :s.shared_ff]
                    v = W @ self._get(map_act, s.shared_act, s.shared_ff)
                y += _sig(z[n]) * v
            o = s.out + r * s.out_stride
            self._put(map_act, o, y + (self._get(map_act, o, E) if s.epi else 0.0))

    def embed_bigram_dev(self, map_act, map_src, h, locs, n_seq, rows, seq0, pos, post=False):
        s = self._spec(h, _BIGRAM)
        toks = self._get(map_act, 0, self.maps[map_act].n)[self.res[locs].view(np.uint32)[:n_seq * rows]].astype(np.int64)
        for r, slot, p in self._tokens(n_seq, rows, seq0, pos):
            at = slot * s.seq_stride + s.prev_off
            pair = (int(self._get(s.state_map, at, 1)[0]) * s.mul_prev + int(toks[r]) * s.mul_cur) % s.buckets if p else s.buckets
            self._put(s.state_map, at, [toks[r]])
            self._put(map_act, s.dst + r * s.width, self._get(map_src, s.table + int(toks[r]) * s.width, s.width) * s.scale
                      + self._get(map_src, s.pairs + pair * s.width, s.width))
