"""A block model on the device with one session, stepped in portions, and how far results are from what is wanted."""
import numpy as np


class Device:
    """a model and one session of it; closes both"""

    def __init__(self, lva, model, backlog=512):
        self.model = model
        self.sess = lva.Session(self.model, backlog)
        self.sess.keep_all_logits(True)

    def close(self):
        self.sess.close()
        self.model.close()

    def __enter__(self):
        return self

    def __exit__(self, *a):
        self.close()

    def step(self, tokens, pos):
        self.sess.begin(tokens, pos)
        return self.sess.logits_rows(0, len(tokens))

    def run(self, tokens, cuts):
        """tokens in portions of the given sizes (the last size repeats)"""
        out, pos, i = [], 0, 0
        while pos < len(tokens):
            n = min(cuts[min(i, len(cuts) - 1)], len(tokens) - pos)
            out.append(self.step(tokens[pos:pos + n], pos))
            pos += n
            i += 1
        return np.concatenate(out)


def rel(got, want):
    """root mean square of the difference, row by row, against the rows' own"""
    d = np.sqrt(np.mean((got - want) ** 2, axis=-1))
    return float(np.max(d / np.sqrt(np.mean(np.asarray(want) ** 2))))


def tokens_for(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.uint32)
