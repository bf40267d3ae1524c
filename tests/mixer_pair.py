"""One op on the HIP library and on the NumPy surface: the same maps, the same handles, results side by side."""
import numpy as np

import oracle
from adam_amd import adamah as A

WS, OP, WT, ST, CA = 0, 2, 1, 3, 14


class Pair:
    """The same maps and handles on the HIP library and on the NumPy surface."""

    def __init__(self, hip, ws, wt=64, opnd=64, state=64, cache=64, dtype="float32"):
        self.g = (hip, oracle.init())
        wide = A.DTYPE_F32 if dtype == "float32" else A.DTYPE_BF16
        for g in self.g:
            for mid, dt, n in ((WS, A.DTYPE_F32, ws), (WT, A.DTYPE_BF16, wt), (OP, wide, opnd), (ST, A.DTYPE_F32, state), (CA, wide, cache)):
                g.map_create_typed(mid, dt, 1, n)
            g.set_dtype(A.DTYPE_F32)
        self.n = ws

    def put(self, mid, off, v):
        v = np.asarray(v)
        v = np.ascontiguousarray(v if v.dtype == np.uint16 else v.astype(np.float32)).reshape(-1)
        for g in self.g:
            g.scatter_contiguous(mid, off, v)

    def up(self, words):
        return tuple(g.upload_dev(np.ascontiguousarray(words, np.uint32))[0] for g in self.g)

    def call(self, name, *args):
        """Handles are pairs (one per side)."""
        for i, g in enumerate(self.g):
            getattr(g, name)(*(a[i] if isinstance(a, tuple) else a for a in args))

    def read(self, mid, off, n):
        return [g.gather(mid, np.arange(off, off + n, dtype=np.uint32)).view(np.float32).astype(np.float64) for g in self.g]

    def same(self, mid, off, n, tol, what=""):
        a, b = self.read(mid, off, n)
        assert np.all(np.isfinite(a)), what
        e = np.abs(a - b).max() / max(np.sqrt(np.mean(b * b)), 1e-30)
        assert e < tol, f"{what}: {e}"
