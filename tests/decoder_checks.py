"""What the tests of the decoders opened from a model folder share: running them and comparing rows of logits."""
import numpy as np
from rikanex_models import write_folder


def row_errors(got, want):
    """Of each row, the root mean square of the difference over that of all wanted rows."""
    return np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want**2).mean())


def rows_close(got, want, limit, share=0.0):
    """-> (are all rows but a share of them within the limit?, text)"""
    e = row_errors(got, want)
    over = int((e > limit).sum())
    ok = bool(np.isfinite(e).all() and over <= share * len(e))
    return ok, f"{over} of {len(e)} rows over the limit, worst {int(e.argmax())}: {e.max():.2e}"


def opened(moon, ctx, path, dtype, max_seq=512):
    return moon.registry.open_text_model(str(path), dtype, max_seq, ctx)


def feed(m, ids, portions):
    """Logits of all tokens, fed in portions."""
    out, at, i = [], 0, 0
    while at < len(ids):
        n = min(portions[i % len(portions)], len(ids) - at)
        out.append(m.forward_logits(ids[at:at + n], np.arange(n)))
        at, i = at + n, i + 1
    return np.concatenate(out)


def run(moon, ctx, tmp_path, cfg, w, ids, dtype, portions=None, max_seq=512):
    """The same with a session of its own (default: all tokens at once)."""
    m = opened(moon, ctx, write_folder(tmp_path / "run", cfg, w), dtype, max_seq)
    got = feed(m, ids, portions or [len(ids)])
    m.close()
    return got
