"""Engine of the layered mixer models (`models.MixerConfig`): bfloat16 weights, float32 residual and state.

It is a `DecodeEngine` whose layers are lists of mixer ops instead of the attention block: generation, sampling modes,
token lookahead, chunked prefill, lockstep batches and decode plans are the base class's; this class lays out weights,
row buffers, state and cache, and issues the ops.  The op list is made once (`_program`); a step runs it with the
number of rows and the position filled in, from Python or as a registered decode plan.

Maps: 0 float32 workspace (rows, small parameters), 1 and up bfloat16 weights (rows padded to a multiple of 64 with
zeros), 2 operand rows of multi-row products, 3 float32 recurrent state, 14 key-value cache.
`dtype='bfloat16'`: operand rows and cache in bfloat16.  'float32': both in float32 and every product in float32; the
weights are stored in bfloat16 either way, which is exact for a model file that holds them so.

What a sequence keeps is bounded: recurrent state, convolution inputs and one attention chunk per layer, so there is
no cache length to choose and no end to a sequence (positions count up to 2^24, where float32 angles stop being exact).
"""
import numpy as np

from .engine import DecodeEngine
from .safetensors_file import TensorDict


def _up_to(n, m):
    return (n + m - 1) // m * m


class SequenceSlots:
    """Which slot of the state and cache a named sequence has, and how many of its tokens the slot holds.  A slot that
    is given back can be handed out again as it is: a sequence's first token reads nothing of it."""

    def __init__(self, n):
        self.pos = [0] * n
        self._free = list(range(n))
        self._of = {}

    def open(self, name):
        if name not in self._of:
            if not self._free:
                raise RuntimeError(f"all {len(self.pos)} sequence slots are in use")
            s = self._of[name] = self._free.pop(0)
            self.pos[s] = 0
        return self._of[name]

    def close(self, name):
        if name in self._of:
            self._free.append(self._of.pop(name))

    def reset(self):
        self.__init__(len(self.pos))


class MixerEngine(DecodeEngine):
    OPND_MAP, STATE_MAP, CACHE_MAP = 2, 3, 14
    WEIGHT_MAPS = [1] + list(range(4, 14))
    LOGIT_ROWS = 16                 # rows of logits a scoring step computes at a time
    MAX_POS = 1 << 24

    def __init__(self, gpu, cfg, tensors, A=None, dtype="bfloat16", prefill_chunk=512, batch=1, map_elem_limit=(1 << 32) - (1 << 24),
                 decode_plan=True, plan_id=0, lookahead=True, sampling_mode=None, **kw):
        if dtype not in ("bfloat16", "float32"):
            raise ValueError(f"dtype '{dtype}': bfloat16 or float32")
        self.dtype = dtype
        self._map_limit = int(map_elem_limit)
        self._kept = 0
        if isinstance(tensors, dict):
            tensors = TensorDict(tensors)
        super().__init__(gpu, cfg, tensors, A=A, kv_cap=self.MAX_POS, fusion_scheduler_mode='level_batched',
                         decode_plan=decode_plan, plan_id=plan_id, prefill_chunk=max(1, int(prefill_chunk)), batch=batch,
                         lookahead=lookahead, sampling_mode=sampling_mode, **kw)

    # ------------------------------------------------------------------ layout
    def _take_tensors(self, tensors):
        return tensors

    def _build_layout(self):
        """Weight matrices -> (map, offset, rows, columns, stride); what shares an input is stacked.  Shapes are checked
        against the configuration, so that a wrong file fails here and by name."""
        c, t = self.cfg, self.tensors
        for name, want in c.tensors().items():
            if name not in t:
                raise ValueError(f"model file lacks tensor {name}")
            have = t.shape(name)
            if len(have) != len(want) or any(w is not None and w != h for w, h in zip(want, have)):
                raise ValueError(f"tensor {name} has shape {have}, expected {want}")
        self._tied, self._lm_name, self._kind = False, 'head', {'head': 'bf16'}
        self._stacks = {}               # stack key (tuple of names) -> (map, offset, n, k, stride)
        self._pack = []                 # (map, offset, kind, names)
        self._map_size = {}
        where = [0, 0]                  # weight map index, position

        def place(groups):
            total = sum(g[2] * g[4] for g in groups)
            if where[1] and where[1] + total > self._map_limit:
                where[:] = [where[0] + 1, 0]
            if where[0] >= len(self.WEIGHT_MAPS):
                raise MemoryError("the model's weights exceed the weight maps")
            for key, kind, n, k, stride in groups:
                mid = self.WEIGHT_MAPS[where[0]]
                self._stacks[key] = (mid, where[1], n, k, stride)
                self._pack.append((mid, where[1], kind, key, n, k, stride))
                where[1] += n * stride
                self._map_size[mid] = where[1]

        def stack(names):
            k = t.shape(names[0])[1]
            if any(t.shape(n)[1] != k for n in names):
                raise ValueError(f"stacked tensors differ in width: {names}")
            return (tuple(names), 'rows', sum(t.shape(n)[0] for n in names), k, _up_to(k, 64))

        E = c.n_embd
        place([(('embed',), 'dense', c.n_vocab, E, E)])
        where[1] = self._map_size[self.WEIGHT_MAPS[where[0]]] = _up_to(where[1], 64)
        place([stack(['head'])])
        self._ff_stride = {}
        for i, L in enumerate(c.layers):
            p = f'l{i}.mix.'
            vec = set(L.mixer.vectors())
            ins = [p + n for n in L.mixer.inputs()]
            rest = [p + n for n, s in L.mixer.tensors(E).items() if len(s) == 2 and n not in vec and p + n not in ins]
            groups = [stack(ins)] + [stack([n]) for n in rest]
            if L.ff:
                m = f'l{i}.mlp.'
                groups.append(((m + 'gate', m + 'up'), 'pairs', 2 * _up_to(L.ff, 16), E, _up_to(E, 64)))
                groups.append(stack([m + 'down']))
            place(groups)
        self._vec_names = ['final.norm']
        for i, L in enumerate(c.layers):
            self._vec_names += [f'l{i}.norm1'] + ([f'l{i}.norm2'] if L.ff else []) + [f'l{i}.mix.{n}' for n in L.mixer.vectors()]
        if self.dtype == "float32":
            bad = [n for g in self._pack for n in g[3] if not t.is_bf16_exact(n)]
            if bad:
                raise ValueError(f"dtype float32: tensor {bad[0]} does not fit bfloat16 storage without rounding")
        self._map_of = {'head': self._stacks[('head',)][0]}

    # ------------------------------------------------------------------ workspace
    def _alloc_workspace(self):
        c, M, E = self.cfg, self._chunk, self.cfg.n_embd
        self._ws = {}
        self._fused_groups = 1
        self._c1, self._c_tok1 = {}, None
        pos = 0

        def take(n, align=64):
            nonlocal pos
            pos = _up_to(pos, align)
            pos += n
            return pos - n

        # rows: every buffer holds M rows, as wide as the widest layer needs
        width = {"hidden": E}
        shape = lambda n: self.tensors.shape(n)
        ff = [L.ff for L in c.layers if L.ff]
        for i, L in enumerate(c.layers):
            p = f'l{i}.mix.'
            w = dict(L.mixer.widths(lambda n: shape(p + n)))
            w["x"] = sum(shape(p + n)[0] for n in L.mixer.inputs())
            for n, v in w.items():
                width[n] = max(width.get(n, 0), E if v is None else v)
        self._rows = {}
        for n, w in width.items():
            w = w if n == "hidden" else _up_to(w, 4)      # (the embedding op writes its rows back to back)
            self._rows[n] = (take(M * w), w)
        self._rows["act"] = (take(_up_to(max(ff, default=0), 16)), _up_to(max(ff, default=0), 16))
        self._rows["logit_rows"] = (take(max(self.LOGIT_ROWS, self._batch) * c.n_vocab), c.n_vocab)
        for name, sz in self._sample_slots():
            self._span(name, sz, take(sz))
        self._rows["logits"] = (self._ws['logits'][2], c.n_vocab)
        self._ws['hidden'] = self._ws['normed'] = (0, E, self._rows["hidden"][0])
        self._c_tok_pos = take(M)
        self._c_tok_locs = np.arange(self._c_tok_pos, self._c_tok_pos + M, dtype=np.uint32)
        self._tok_rows_h = self._up(self._c_tok_locs)
        self._hid_locs = np.arange(self._rows["hidden"][0], self._rows["hidden"][0] + E, dtype=np.uint32)
        self._alloc_sample_handles()
        self._vec_off = {n: take(int(np.prod(self.tensors.shape(n)))) for n in self._vec_names}
        self._consts = {}
        self._const_at = take(sum(L.mixer.const_size() for L in c.layers))
        self._ws_total = pos
        # operand rows: one region for what a product normalises or converts, one per feed-forward width
        kmax = max(s[4] for k, s in self._stacks.items() if k != ('embed',))
        self._opnd_total = M * kmax
        self._act_opnd = {}
        for f in sorted(set(ff)):
            self._act_opnd[f] = self._opnd_total
            self._opnd_total += M * _up_to(f, 64)
        self.state_per_seq = _up_to(sum(L.mixer.state_size() for L in c.layers), 64) or 64
        self.cache_per_seq = _up_to(sum(L.mixer.cache_size() for L in c.layers), 64) or 64
        self.slots = SequenceSlots(self._batch)

    # ------------------------------------------------------------------ upload
    def _upload_all(self):
        g, A, t = self.gpu, self.A, self.tensors
        g.set_dtype(A.DTYPE_F32)
        g.map_create(self.WS_MAP, 1, self._ws_total)
        wide = A.DTYPE_F32 if self.dtype == "float32" else A.DTYPE_BF16
        g.map_create_typed(self.OPND_MAP, wide, 1, self._opnd_total)
        g.map_create_typed(self.STATE_MAP, A.DTYPE_F32, 1, self._batch * self.state_per_seq)
        g.map_create_typed(self.CACHE_MAP, wide, 1, self._batch * self.cache_per_seq)
        for mid, n in self._map_size.items():
            g.map_create_typed(mid, A.DTYPE_BF16, 1, n)
        step = 1 << 24

        def put(mid, off, rows):
            flat = np.ascontiguousarray(rows).reshape(-1)
            for b in range(0, flat.size, step):
                g.scatter_contiguous(mid, off + b, flat[b:b + step])

        for mid, off, kind, names, n, k, stride in self._pack:
            if kind == 'pairs':                          # 16 gate rows, their 16 up rows, and so on
                ff = t.shape(names[0])[0]
                block = np.zeros((n // 32, 2, 16, stride), np.uint16)
                for j, name in enumerate(names):
                    w = np.zeros((n // 2, stride), np.uint16)
                    w[:ff, :k] = t.bf16(name)
                    block[:, j] = w.reshape(n // 32, 16, stride)
                put(mid, off, block)
                continue
            for name in names:
                w = t.bf16(name)
                if stride != k:
                    pad = np.zeros((w.shape[0], stride), np.uint16)
                    pad[:, :k] = w
                    w = pad
                put(mid, off, w)
                off += w.shape[0] * stride
        for n, off in self._vec_off.items():
            g.scatter_contiguous(self.WS_MAP, off, np.ascontiguousarray(t.f32(n)).reshape(-1))

    def _alloc_kv_cache(self):
        self.reset()

    def _upload_locs(self):
        self._program = []
        self._state_at = self._cache_at = 0
        self._emit = self._program
        for i, L in enumerate(self.cfg.layers):
            p = f'l{i}.mix.'
            ins = [p + n for n in L.mixer.inputs()]
            cols, at = {}, 0
            for n in L.mixer.inputs():
                cols[n] = at
                at += self.tensors.shape(p + n)[0]
            self.linear(ins, src=self.at("hidden"), out=self.at("x"), norm=self.model_norm(f'l{i}.norm1'))
            L.mixer.core(self, p, cols)
            L.mixer.output(self, p, cols, self.at("hidden"), self.A.EPI_ADD)
            if L.ff:
                self._feed_forward(i, L.ff)
        self._heads, self._row_lists = {}, {}
        self._score_h = self._head_spec(0, "logit_rows")

    def _feed_forward(self, i, ff):
        A, m = self.A, f'l{i}.mlp.'
        act = (self._act_opnd[ff], _up_to(ff, 64))
        self.linear([m + 'gate', m + 'up'], src=self.at("hidden"), out=self.at("act"), norm=self.model_norm(f'l{i}.norm2'),
                    epi=A.EPI_SWIGLU, out_opnd=act)
        self.linear([m + 'down'], src=self.at("act"), out=self.at("hidden"), epi=A.EPI_ADD, opnd=act[0], ready=1)

    # ------------------------------------------------------------------ what mixers issue their ops through
    def at(self, rows, col=0):
        """(offset, stride) of a row buffer, from column `col` on."""
        off, stride = self._rows[rows]
        return off + col, stride

    def vec(self, name):
        return self._vec_off[name]

    def const(self, values):
        """Workspace offset of float32 constants (kept once per distinct list)."""
        v = np.asarray(values, np.float64).astype(np.float32)
        key = v.tobytes()
        if key not in self._consts:
            self._consts[key] = self._const_at
            if v.size:
                self.gpu.scatter_contiguous(self.WS_MAP, self._const_at, v)
            self._const_at += v.size
        return self._consts[key]

    def take_state(self, n):
        self._state_at += n
        return self._state_at - n

    def take_cache(self, n):
        self._cache_at += n
        return self._cache_at - n

    @staticmethod
    def norm(groups, wt=0, wt_len=0, gate=None, eps=None):
        d = {"groups": groups, "wt": wt, "wt_len": wt_len, "eps": eps}
        if gate is not None:
            d.update(gate=gate[0], gate_stride=gate[1], gate_act=gate[2])
        return d

    def model_norm(self, name):
        return self.norm(self.cfg.norm_groups, self.vec(name), self.cfg.n_embd)

    def linear_spec(self, names, src, out, norm=None, epi=0, opnd=0, ready=0, out_opnd=(0, 0)):
        """(weight map, spec handle) of y = W . f(x)."""
        mid, off, n, k, stride = self._stacks[tuple(names)]
        f = dict(norm or {"groups": 0})
        f["eps"] = self.cfg.norm_eps if f.get("eps") is None else f["eps"]
        spec = self.A.LinearSpec(w=off, n=n, k=k, k_stride=stride, src=src[0], src_stride=src[1], opnd=opnd, ready=ready, out=out[0],
                                 out_stride=out[1], epi=epi, out_opnd=out_opnd[0], out_opnd_stride=out_opnd[1], **f)
        return mid, self._up(spec.words())

    def linear(self, names, src, out, **kw):
        mid, h = self.linear_spec(names, src, out, **kw)
        self._emit.append((self.A.DECODE_OP_LINEAR, mid, h, 0, 0))

    def delta_rule(self, spec, decay, gate):
        assert decay[0] == gate[0]
        self._emit.append((self.A.DECODE_OP_DELTA_RULE, decay[0], self._up(spec.words()), decay[1], gate[1]))

    def retention(self, spec):
        self._emit.append((self.A.DECODE_OP_RETENTION, 0, self._up(spec.words()), 0, 0))

    def chunk_attention(self, spec):
        self._emit.append((self.A.DECODE_OP_CHUNK_ATTENTION, 0, self._up(spec.words()), 0, 0))

    def merge(self, a, b, wa, wb, out, scale):
        ao, stride = self.at(a)
        bo, stride_b = self.at(b)
        assert stride == stride_b
        spec = self.A.MergeSpec(a=ao, b=bo, stride=stride, wa=wa, wb=wb, dst=out[0], dst_stride=out[1], dim=self.cfg.n_embd,
                                eps=self.cfg.norm_eps, scale=scale)
        self._emit.append((self.A.DECODE_OP_MERGE_NORM, 0, self._up(spec.words()), 0, 0))

    # ------------------------------------------------------------------ running the op list
    def _run_program(self, n_seq, rows, seq0, pos):
        """`rows` tokens of one sequence, or one token of each of n_seq sequences, from the hidden rows to the hidden rows."""
        g, A, ws, n = self.gpu, self.A, self.WS_MAP, n_seq * rows
        for kind, mid, h0, h1, h2 in self._program:
            if kind == A.DECODE_OP_LINEAR:
                g.linear_dev(ws, self.OPND_MAP, mid, h0, 0, n)
            elif kind == A.DECODE_OP_MERGE_NORM:
                g.merge_norm_dev(ws, h0, n)
            elif kind == A.DECODE_OP_DELTA_RULE:
                g.delta_rule_dev(ws, self.OPND_MAP, mid, h0, h1, h2, n_seq, rows, seq0, pos)
            elif kind == A.DECODE_OP_RETENTION:
                g.retention_dev(ws, h0, n_seq, rows, seq0, pos)
            else:
                g.chunk_attention_dev(ws, h0, n_seq, rows, seq0, pos)

    def _ops_for(self, n_seq):
        A, P = self.A, self.A.DECODE_RUNTIME_POS
        ops = []
        for kind, mid, h0, h1, h2 in self._program:
            op = A.DecodePlanOp(kind=kind, map_id=self.WS_MAP, map_id2=mid, op_code=self.OPND_MAP, h0=h0, h1=h1, h2=h2, u0=n_seq)
            if kind not in (A.DECODE_OP_LINEAR, A.DECODE_OP_MERGE_NORM):
                op.u1, op.u2, op.u3 = 1, 0, P
            ops.append(op)
        return ops

    def _plan_ops(self):
        return self._ops_for(1)

    def _lockstep_plan_ops(self, m):
        return self._ops_for(m)

    # ------------------------------------------------------------------ steps
    def _head_spec(self, row, out):
        src, stride = self.at("hidden")
        return self.linear_spec(['head'], src=(src + row * stride, stride), out=self.at(out), norm=self.model_norm('final.norm'))

    def _head(self, row):
        """Spec handle of final norm and LM head over hidden row `row`, logits to the `logits` slot."""
        if row not in self._heads:
            self._heads[row] = self._head_spec(row, "logits")
        return self._heads[row]

    def _advance(self, slot, pos, n):
        if self.slots.pos[slot] != pos:
            raise RuntimeError(f"sequence slot {slot} holds {self.slots.pos[slot]} tokens; a step at position {pos} cannot follow")
        if pos + n > self.MAX_POS:
            raise RuntimeError(f"sequence of {pos + n} tokens: at most {self.MAX_POS}")
        self.slots.pos[slot] = pos + n

    def _token_feed(self):
        if self._feed is None:
            mid, off = self._stacks[('embed',)][:2]
            self._feed = {'src': (mid, off), 'tok_h': self._up(self._sample_locs), 'tok_hs': {self._batch: self._tok_rows_h}}
        return self._feed

    def _check_tokens(self, toks):
        toks = np.asarray(toks, np.int64)
        if toks.size and (toks.min() < 0 or toks.max() >= self.cfg.n_vocab):
            raise ValueError(f"token ids must lie in 0 .. {self.cfg.n_vocab - 1}")
        return toks.astype(np.float32)

    def _embed(self, toks):
        c, feed = self.cfg, self._token_feed()
        self.gpu.scatter_contiguous(self.WS_MAP, self._c_tok_pos, self._check_tokens(toks))
        self.gpu.embed_tokens_dev(self.WS_MAP, feed['src'][0], self._tok_rows_h, feed['src'][1], self._rows["hidden"][0], len(toks),
                                  c.n_embd, c.n_vocab, 1.0)

    def _stage_token(self, tok, from_device):
        self._next = None if from_device else tok

    def _issue_embedding(self, from_device):
        c, feed = self.cfg, self._token_feed()
        if not from_device:
            return self._embed([self._next])
        self._feed_ticket = self.gpu.embed_post_tokens_dev(self.WS_MAP, feed['src'][0], feed['tok_h'], feed['src'][1],
                                                           self._rows["hidden"][0], 1, c.n_embd, c.n_vocab, 1.0)

    def _issue_layers(self, pos):
        self._advance(0, pos, 1)
        if self._plan_id is not None:
            self.gpu.decode_step(self._plan_id, pos, pos + 1)
        else:
            self._run_program(1, 1, 0, pos)

    def _issue_argmax(self, normed_h):
        mid, h = self._head(0)
        self.gpu.linear_argmax_dev(self.WS_MAP, self.OPND_MAP, mid, h, self._feed['tok_h'], 1)

    def _issue_logits(self, normed_h):
        mid, h = self._head(0)
        self.gpu.linear_dev(self.WS_MAP, self.OPND_MAP, mid, h, 0, 1)

    def _head_argmax_built(self):
        return hasattr(self.gpu, 'linear_argmax_dev')

    def _forward_chunk(self, toks, pos0, sample=True, seq=0, lockstep=False, from_device=False):
        """m prompt tokens of sequence `seq` at positions pos0 .. in one pass, or (`lockstep`) one token of each of the
        first m sequences, all at position pos0; see the base class."""
        c, g, ws = self.cfg, self.gpu, self.WS_MAP
        m = self._batch if from_device else len(toks)
        if m == 0 or m > self._chunk:
            raise RuntimeError(f"chunk of {m} tokens does not fit prefill_chunk={self._chunk}")
        g.batch_begin()
        if from_device:
            feed = self._token_feed()
            self._feed_ticket = g.embed_post_tokens_dev(ws, feed['src'][0], feed['tok_hs'][m], feed['src'][1], self._rows["hidden"][0],
                                                        m, c.n_embd, c.n_vocab, 1.0)
        else:
            self._embed(toks)
        for s in range(m if lockstep else 1):
            self._advance(s if lockstep else seq, pos0, 1 if lockstep else m)
        if lockstep and self._ls_plan_id is not None and m == self._batch:
            g.decode_step(self._ls_plan_id, pos0, pos0 + 1)
        elif lockstep:
            self._run_program(m, 1, 0, pos0)
        else:
            self._run_program(1, m, seq, pos0)
        if lockstep:
            mid, h = self._score_h
            g.linear_argmax_dev(ws, self.OPND_MAP, mid, h, self._tok_rows_h, m)
        elif sample:
            mid, h = self._head(m - 1)
            g.linear_argmax_dev(ws, self.OPND_MAP, mid, h, self._feed['tok_h'], 1)
            self._sample_token_ready = True
        g.batch_end()

    def reset(self):
        self.__init__(len(self.pos))


class MixerEngine(DecodeEngine):
    OPND_MAP, STATE_MAP, CACHE_MAP = 2, 3, 14
    WEIGHT_MAPS = [1] + list(range(4, 14))
    LOGIT_ROWS = 16                 # rows of logits a scoring step computes at a time
    MAX_POS = 1 << 24

    def __init__(self, gpu, cfg, tensors, A=None, dtype="bfloat16", prefill_chunk=512, batch=1, map_elem_limit=(1 << 32) - (1 << 24),
                 decode_plan=True, plan_id=0, lookahead=True, sampling_mode=None, **kw):
        if dtype not in ("bfloat16", "float32"):
            raise ValueError(f"dtype '{dtype}': bfloat16 or float32")
        self.dtype = dtype
        self._map_limit = int(map_elem_limit)
        self._kept = 0
        if isinstance(tensors, dict):
            tensors = TensorDict(tensors)
        super().__init__(gpu, cfg, tensors, A=A, kv_cap=self.MAX_POS, fusion_scheduler_mode='level_batched',
                         decode_plan=decode_plan, plan_id=plan_id, prefill_chunk=max(1, int(prefill_chunk)), batch=batch,
                         lookahead=lookahead, sampling_mode=sampling_mode, **kw)

    # ------------------------------------------------------------------ layout
    def _take_tensors(self, tensors):
        return tensors

    def _build_layout(self):
        """Weight matrices -> (map, offset, rows, columns, stride); what shares an input is stacked.  Shapes are checked
        against the configuration, so that a wrong file fails here and by name."""
        c, t = self.cfg, self.tensors
        for name, want in c.tensors().items():
            if name not in t:
                raise ValueError(f"model file lacks tensor {name}")
            have = t.shape(name)
            if len(have) != len(want) or any(w is not None and w != h for w, h in zip(want, have)):
                raise ValueError(f"tensor {name} has shape {have}, expected {want}")
        self._tied, self._lm_name, self._kind = False, 'head', {'head': 'bf16'}
        self._stacks = {}               # stack key (tuple of names) -> (map, offset, n, k, stride)
        self._pack = []                 # (map, offset, kind, names)
        self._map_size = {}
        where = [0, 0]                  # weight map index, position

        def place(groups):
            total = sum(g[2] * g[4] for g in groups)
            if where[1] and where[1] + total > self._map_limit:
                where[:] = [where[0] + 1, 0]
            if where[0] >= len(self.WEIGHT_MAPS):
                raise MemoryError("the model's weights exceed the weight maps")
            for key, kind, n, k, stride in groups:
                mid = self.WEIGHT_MAPS[where[0]]
                self._stacks[key] = (mid, where[1], n, k, stride)
                self._pack.append((mid, where[1], kind, key, n, k, stride))
                where[1] += n * stride
                self._map_size[mid] = where[1]

        def stack(names):
            k = t.shape(names[0])[1]
            if any(t.shape(n)[1] != k for n in names):
                raise ValueError(f"stacked tensors differ in width: {names}")
            return (tuple(names), 'rows', sum(t.shape(n)[0] for n in names), k, _up_to(k, 64))

        E = c.n_embd
        place([(('embed',), 'dense', c.n_vocab, E, E)])
        where[1] = self._map_size[self.WEIGHT_MAPS[where[0]]] = _up_to(where[1], 64)
        place([stack(['head'])])
        self._ff_stride = {}
        for i, L in enumerate(c.layers):
            p = f'l{i}.mix.'
            vec = set(L.mixer.vectors())
            ins = [p + n for n in L.mixer.inputs()]
            rest = [p + n for n, s in L.mixer.tensors(E).items() if len(s) == 2 and n not in vec and p + n not in ins]
            groups = [stack(ins)] + [stack([n]) for n in rest]
            if L.ff:
                m = f'l{i}.mlp.'
                groups.append(((m + 'gate', m + 'up'), 'pairs', 2 * _up_to(L.ff, 16), E, _up_to(E, 64)))
                groups.append(stack([m + 'down']))
            place(groups)
        self._vec_names = ['final.norm']
        for i, L in enumerate(c.layers):
            self._vec_names += [f'l{i}.norm1'] + ([f'l{i}.norm2'] if L.ff else []) + [f'l{i}.mix.{n}' for n in L.mixer.vectors()]
        if self.dtype == "float32":
            bad = [n for g in self._pack for n in g[3] if not t.is_bf16_exact(n)]
            if bad:
                raise ValueError(f"dtype float32: tensor {bad[0]} does not fit bfloat16 storage without rounding")
        self._map_of = {'head': self._stacks[('head',)][0]}

    # ------------------------------------------------------------------ workspace
    def _alloc_workspace(self):
        c, M, E = self.cfg, self._chunk, self.cfg.n_embd
        self._ws = {}
        self._fused_groups = 1
        self._c1, self._c_tok1 = {}, None
        pos = 0

        def take(n, align=64):
            nonlocal pos
            pos = _up_to(pos, align)
            pos += n
            return pos - n

        # rows: every buffer holds M rows, as wide as the widest layer needs
        width = {"hidden": E}
        shape = lambda n: self.tensors.shape(n)
        ff = [L.ff for L in c.layers if L.ff]
        for i, L in enumerate(c.layers):
            p = f'l{i}.mix.'
            w = dict(L.mixer.widths(lambda n: shape(p + n)))
            w["x"] = sum(shape(p + n)[0] for n in L.mixer.inputs())
            for n, v in w.items():
                width[n] = max(width.get(n, 0), E if v is None else v)
        self._rows = {}
        for n, w in width.items():
            w = w if n == "hidden" else _up_to(w, 4)      # (the embedding op writes its rows back to back)
            self._rows[n] = (take(M * w), w)
        self._rows["act"] = (take(_up_to(max(ff, default=0), 16)), _up_to(max(ff, default=0), 16))
        self._rows["logit_rows"] = (take(max(self.LOGIT_ROWS, self._batch) * c.n_vocab), c.n_vocab)
        for name, sz in self._sample_slots():
            self._span(name, sz, take(sz))
        self._rows["logits"] = (self._ws['logits'][2], c.n_vocab)
        self._ws['hidden'] = self._ws['normed'] = (0, E, self._rows["hidden"][0])
        self._c_tok_pos = take(M)
        self._c_tok_locs = np.arange(self._c_tok_pos, self._c_tok_pos + M, dtype=np.uint32)
        self._tok_rows_h = self._up(self._c_tok_locs)
        self._hid_locs = np.arange(self._rows["hidden"][0], self._rows["hidden"][0] + E, dtype=np.uint32)
        self._alloc_sample_handles()
        self._vec_off = {n: take(int(np.prod(self.tensors.shape(n)))) for n in self._vec_names}
        self._consts = {}
        self._const_at = take(sum(2 * (getattr(m, 'rot_dims', 0) + len(getattr(m, 'decay', ())) + 64)
                                  for L in c.layers for m in (L.mixer, getattr(L.mixer, 'right', None), getattr(L.mixer, 'left', None)) if m))
        self._ws_total = pos
        # operand rows: one region for what a product normalises or converts, one per feed-forward width
        kmax = max(s[4] for k, s in self._stacks.items() if k != ('embed',))
        self._opnd_total = M * kmax
        self._act_opnd = {}
        for f in sorted(set(ff)):
            self._act_opnd[f] = self._opnd_total
            self._opnd_total += M * _up_to(f, 64)
        self.state_per_seq = _up_to(sum(L.mixer.state_size() for L in c.layers), 64) or 64
        self.cache_per_seq = _up_to(sum(L.mixer.cache_size() for L in c.layers), 64) or 64
        self.slots = SequenceSlots(self._batch)

    # ------------------------------------------------------------------ upload
    def _upload_all(self):
        g, A, t = self.gpu, self.A, self.tensors
        g.set_dtype(A.DTYPE_F32)
        g.map_create(self.WS_MAP, 1, self._ws_total)
        wide = A.DTYPE_F32 if self.dtype == "float32" else A.DTYPE_BF16
        g.map_create_typed(self.OPND_MAP, wide, 1, self._opnd_total)
        g.map_create_typed(self.STATE_MAP, A.DTYPE_F32, 1, self._batch * self.state_per_seq)
        g.map_create_typed(self.CACHE_MAP, wide, 1, self._batch * self.cache_per_seq)
        for mid, n in self._map_size.items():
            g.map_create_typed(mid, A.DTYPE_BF16, 1, n)
        step = 1 << 24

        def put(mid, off, rows):
            flat = np.ascontiguousarray(rows).reshape(-1)
            for b in range(0, flat.size, step):
                g.scatter_contiguous(mid, off + b, flat[b:b + step])

        for mid, off, kind, names, n, k, stride in self._pack:
            if kind == 'pairs':                          # 16 gate rows, their 16 up rows, and so on
                ff = t.shape(names[0])[0]
                block = np.zeros((n // 32, 2, 16, stride), np.uint16)
                for j, name in enumerate(names):
                    w = np.zeros((n // 2, stride), np.uint16)
                    w[:ff, :k] = t.bf16(name)
                    block[:, j] = w.reshape(n // 32, 16, stride)
                put(mid, off, block)
                continue
            for name in names:
                w = t.bf16(name)
                if stride != k:
                    pad = np.zeros((w.shape[0], stride), np.uint16)
                    pad[:, :k] = w
                    w = pad
                put(mid, off, w)
                off += w.shape[0] * stride
        for n, off in self._vec_off.items():
            g.scatter_contiguous(self.WS_MAP, off, np.ascontiguousarray(t.f32(n)).reshape(-1))

    def _alloc_kv_cache(self):
        self.reset()

    def _upload_locs(self):
        self._program = []
        self._state_at = self._cache_at = 0
        self._emit = self._program
        for i, L in enumerate(self.cfg.layers):
            p = f'l{i}.mix.'
            ins = [p + n for n in L.mixer.inputs()]
            cols, at = {}, 0
            for n in L.mixer.inputs():
                cols[n] = at
                at += self.tensors.shape(p + n)[0]
            self.linear(ins, src=self.at("hidden"), out=self.at("x"), norm=self.model_norm(f'l{i}.norm1'))
            L.mixer.core(self, p, cols)
            L.mixer.output(self, p, cols, self.at("hidden"), self.A.EPI_ADD)
            if L.ff:
                self._feed_forward(i, L.ff)
        self._heads, self._row_lists = {}, {}
        self._score_h = self._head_spec(0, "logit_rows")

    def _feed_forward(self, i, ff):
        A, m = self.A, f'l{i}.mlp.'
        act = (self._act_opnd[ff], _up_to(ff, 64))
        self.linear([m + 'gate', m + 'up'], src=self.at("hidden"), out=self.at("act"), norm=self.model_norm(f'l{i}.norm2'),
                    epi=A.EPI_SWIGLU, out_opnd=act)
        self.linear([m + 'down'], src=self.at("act"), out=self.at("hidden"), epi=A.EPI_ADD, opnd=act[0], ready=1)

    # ------------------------------------------------------------------ what mixers issue their ops through
    def at(self, rows, col=0):
        """(offset, stride) of a row buffer, from column `col` on."""
        off, stride = self._rows[rows]
        return off + col, stride

    def vec(self, name):
        return self._vec_off[name]

    def const(self, values):
        """Workspace offset of float32 constants (kept once per distinct list)."""
        v = np.asarray(values, np.float64).astype(np.float32)
        key = v.tobytes()
        if key not in self._consts:
            self._consts[key] = self._const_at
            if v.size:
                self.gpu.scatter_contiguous(self.WS_MAP, self._const_at, v)
            self._const_at += v.size
        return self._consts[key]

    def take_state(self, n):
        self._state_at += n
        return self._state_at - n

    def take_cache(self, n):
        self._cache_at += n
        return self._cache_at - n

    @staticmethod
    def norm(groups, wt=0, wt_len=0, gate=None, eps=None):
        d = {"groups": groups, "wt": wt, "wt_len": wt_len, "eps": eps}
        if gate is not None:
            d.update(gate=gate[0], gate_stride=gate[1], gate_act=gate[2])
        return d

    def model_norm(self, name):
        return self.norm(self.cfg.norm_groups, self.vec(name), self.cfg.n_embd)

    def linear_spec(self, names, src, out, norm=None, epi=0, opnd=0, ready=0, out_opnd=(0, 0)):
        """(weight map, spec handle) of y = W . f(x)."""
        mid, off, n, k, stride = self._stacks[tuple(names)]
        f = dict(norm or {"groups": 0})
        f["eps"] = self.cfg.norm_eps if f.get("eps") is None else f["eps"]
        spec = self.A.LinearSpec(w=off, n=n, k=k, k_stride=stride, src=src[0], src_stride=src[1], opnd=opnd, ready=ready, out=out[0],
                                 out_stride=out[1], epi=epi, out_opnd=out_opnd[0], out_opnd_stride=out_opnd[1], **f)
        return mid, self._up(spec.words())

    def linear(self, names, src, out, **kw):
        mid, h = self.linear_spec(names, src, out, **kw)
        self._emit.append((self.A.DECODE_OP_LINEAR, mid, h, 0, 0))

    def delta_rule(self, spec, decay, gate):
        assert decay[0] == gate[0]
        self._emit.append((self.A.DECODE_OP_DELTA_RULE, decay[0], self._up(spec.words()), decay[1], gate[1]))

    def retention(self, spec):
        self._emit.append((self.A.DECODE_OP_RETENTION, 0, self._up(spec.words()), 0, 0))

    def chunk_attention(self, spec):
        self._emit.append((self.A.DECODE_OP_CHUNK_ATTENTION, 0, self._up(spec.words()), 0, 0))

    def merge(self, a, b, wa, wb, out, scale):
        ao, stride = self.at(a)
        bo, stride_b = self.at(b)
        assert stride == stride_b
        spec = self.A.MergeSpec(a=ao, b=bo, stride=stride, wa=wa, wb=wb, dst=out[0], dst_stride=out[1], dim=self.cfg.n_embd,
                                eps=self.cfg.norm_eps, scale=scale)
        self._emit.append((self.A.DECODE_OP_MERGE_NORM, 0, self._up(spec.words()), 0, 0))

    # ------------------------------------------------------------------ running the op list
    def _run_program(self, n_seq, rows, seq0, pos):
        """`rows` tokens of one sequence, or one token of each of n_seq sequences, from the hidden rows to the hidden rows."""
        g, A, ws, n = self.gpu, self.A, self.WS_MAP, n_seq * rows
        for kind, mid, h0, h1, h2 in self._program:
            if kind == A.DECODE_OP_LINEAR:
                g.linear_dev(ws, self.OPND_MAP, mid, h0, 0, n)
            elif kind == A.DECODE_OP_MERGE_NORM:
                g.merge_norm_dev(ws, h0, n)
            elif kind == A.DECODE_OP_DELTA_RULE:
                g.delta_rule_dev(ws, self.OPND_MAP, mid, h0, h1, h2, n_seq, rows, seq0, pos)
            elif kind == A.DECODE_OP_RETENTION:
                g.retention_dev(ws, h0, n_seq, rows, seq0, pos)
            else:
                g.chunk_attention_dev(ws, h0, n_seq, rows, seq0, pos)

    def _ops_for(self, n_seq):
        A, P = self.A, self.A.DECODE_RUNTIME_POS
        ops = []
        for kind, mid, h0, h1, h2 in self._program:
            op = A.DecodePlanOp(kind=kind, map_id=self.WS_MAP, map_id2=mid, op_code=self.OPND_MAP, h0=h0, h1=h1, h2=h2, u0=n_seq)
            if kind not in (A.DECODE_OP_LINEAR, A.DECODE_OP_MERGE_NORM):
                op.u1, op.u2, op.u3 = 1, 0, P
            ops.append(op)
        return ops

    def _plan_ops(self):
        return self._ops_for(1)

    def _lockstep_plan_ops(self, m):
        return self._ops_for(m)

    # ------------------------------------------------------------------ steps
    def _head_spec(self, row, out):
        src, stride = self.at("hidden")
        return self.linear_spec(['head'], src=(src + row * stride, stride), out=self.at(out), norm=self.model_norm('final.norm'))

    def _head(self, row):
        """Spec handle of final norm and LM head over hidden row `row`, logits to the `logits` slot."""
        if row not in self._heads:
            self._heads[row] = self._head_spec(row, "logits")
        return self._heads[row]

    def _advance(self, slot, pos, n):
        if self.slots.pos[slot] != pos:
            raise RuntimeError(f"sequence slot {slot} holds {self.slots.pos[slot]} tokens; a step at position {pos} cannot follow")
        if pos + n > self.MAX_POS:
            raise RuntimeError(f"sequence of {pos + n} tokens: at most {self.MAX_POS}")
        self.slots.pos[slot] = pos + n

    def _token_feed(self):
        if self._feed is None:
            mid, off = self._stacks[('embed',)][:2]
            self._feed = {'src': (mid, off), 'tok_h': self._up(self._sample_locs), 'tok_hs': {self._batch: self._tok_rows_h}}
        return self._feed

    def _check_tokens(self, toks):
        toks = np.asarray(toks, np.int64)
        if toks.size and (toks.min() < 0 or toks.max() >= self.cfg.n_vocab):
            raise ValueError(f"token ids must lie in 0 .. {self.cfg.n_vocab - 1}")
        return toks.astype(np.float32)

    def _embed(self, toks):
        c, feed = self.cfg, self._token_feed()
        self.gpu.scatter_contiguous(self.WS_MAP, self._c_tok_pos, self._check_tokens(toks))
        self.gpu.embed_tokens_dev(self.WS_MAP, feed['src'][0], self._tok_rows_h, feed['src'][1], self._rows["hidden"][0], len(toks),
                                  c.n_embd, c.n_vocab, 1.0)

    def _stage_token(self, tok, from_device):
        self._next = None if from_device else tok

    def _issue_embedding(self, from_device):
        c, feed = self.cfg, self._token_feed()
        if not from_device:
            return self._embed([self._next])
        self._feed_ticket = self.gpu.embed_post_tokens_dev(self.WS_MAP, feed['src'][0], feed['tok_h'], feed['src'][1],
                                                           self._rows["hidden"][0], 1, c.n_embd, c.n_vocab, 1.0)

    def _issue_layers(self, pos):
        self._advance(0, pos, 1)
        if self._plan_id is not None:
            self.gpu.decode_step(self._plan_id, pos, pos + 1)
        else:
            self._run_program(1, 1, 0, pos)

    def _issue_argmax(self, normed_h):
        mid, h = self._head(0)
        self.gpu.linear_argmax_dev(self.WS_MAP, self.OPND_MAP, mid, h, self._feed['tok_h'], 1)

    def _issue_logits(self, normed_h):
        mid, h = self._head(0)
        self.gpu.linear_dev(self.WS_MAP, self.OPND_MAP, mid, h, 0, 1)

    def _head_argmax_built(self):
        return hasattr(self.gpu, 'linear_argmax_dev')

    def _forward_chunk(self, toks, pos0, sample=True, seq=0, lockstep=False, from_device=False):
        """m prompt tokens of sequence `seq` at positions pos0 .. in one pass, or (`lockstep`) one token of each of the
        first m sequences, all at position pos0; see the base class."""
        c, g, ws = self.cfg, self.gpu, self.WS_MAP
        m = self._batch if from_device else len(toks)
        if m == 0 or m > self._chunk:
            raise RuntimeError(f"chunk of {m} tokens does not fit prefill_chunk={self._chunk}")
        g.batch_begin()
        if from_device:
            feed = self._token_feed()
            self._feed_ticket = g.embed_post_tokens_dev(ws, feed['src'][0], feed['tok_hs'][m], feed['src'][1], self._rows["hidden"][0],
                                                        m, c.n_embd, c.n_vocab, 1.0)
        else:
            self._embed(toks)
        for s in range(m if lockstep else 1):
            self._advance(s if lockstep else seq, pos0, 1 if lockstep else m)
        if lockstep and self._ls_plan_id is not None and m == self._batch:
            g.decode_step(self._ls_plan_id, pos0, pos0 + 1)
        elif lockstep:
            self._run_program(m, 1, 0, pos0)
        else:
            self._run_program(1, m, seq, pos0)
        if lockstep:
            mid, h = self._score_h
            g.linear_argmax_dev(ws, self.OPND_MAP, mid, h, self._tok_rows_h, m)
        elif sample:
            mid, h = self._head(m - 1)
            g.linear_argmax_dev(ws, self.OPND_MAP, mid, h, self._feed['tok_h'], 1)
            self._sample_token_ready = True
        g.batch_end()

    def _lockstep_head(self):
        if 'rows' not in self._heads:
            if self._batch > self.LOGIT_ROWS:
                raise RuntimeError(f"lockstep batches of at most {self.LOGIT_ROWS} sequences")
            self._heads['rows'] = self._head_spec(0, "logit_rows")
        return self._heads['rows']

    def reset(self):
        keep, self._kept = self._kept, 0
        self.slots.reset()
        self.slots.pos[0] = keep
        self._sample_token_ready = False

    def _usable_prefix(self, n, n_prompt):
        """A recurrent state cannot be wound back: a prefix is kept only if the slot holds exactly its tokens."""
        self._kept = n if 0 < n < n_prompt and self.slots.pos[0] == n else 0
        return self._kept

    # ------------------------------------------------------------------ scoring
    def score(self, name, tokens, want=()):
        """Feed a named sequence its next tokens; the logits [len(want), n_vocab] at the places `want` among them.  The
        sequence gets a slot with its first tokens and keeps it until `release`."""
        slot = self.slots.open(name)
        tokens = [int(t) for t in tokens]
        self._check_tokens(tokens)
        out = np.empty((len(want), self.cfg.n_vocab), np.float32)
        for lo in range(0, len(tokens), self._chunk):
            part = tokens[lo:lo + self._chunk]
            if len(part) == 1 and slot == 0:
                self._forward(part[0], self.slots.pos[slot], sample=False)
            else:
                self._forward_chunk(part, self.slots.pos[slot], sample=False, seq=slot)
            here = [(i, w - lo) for i, w in enumerate(want) if lo <= w < lo + len(part)]
            for b in range(0, len(here), self.LOGIT_ROWS):
                idx = here[b:b + self.LOGIT_ROWS]
                out[[i for i, _ in idx]] = self._logits_of_rows([r for _, r in idx])
        return out

    def release(self, name):
        self.slots.close(name)

    def _logits_of_rows(self, rows):
        g, n = self.gpu, len(rows)
        r = np.asarray(rows, np.uint32)
        if n in self._row_lists:
            g.upload_dev(r, handle=self._row_lists[n])
        else:
            self._row_lists[n] = self._up(r)
        mid, h = self._score_h
        g.linear_dev(self.WS_MAP, self.OPND_MAP, mid, h, self._row_lists[n], n)
        off = self._rows["logit_rows"][0]
        return g.gather(self.WS_MAP, np.arange(off, off + n * self.cfg.n_vocab, dtype=np.uint32)).view(np.float32).reshape(n, -1)

    def read_rows(self, name, n, width=None):
        """The first n rows of a row buffer (tests, debugging)."""
        off, stride = self._rows[name]
        r = self.gpu.gather(self.WS_MAP, np.arange(off, off + n * stride, dtype=np.uint32)).view(np.float32).reshape(n, stride)
        return r[:, :width or stride].copy()
