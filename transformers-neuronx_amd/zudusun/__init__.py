"""The Zudusun design: layers of one norm whose output a mixer and a feed-forward both read, the mixer either softmax
attention and gated linear attention side by side, softmax attention under a sliding window (a norm a head, turned
heads, a one in the softmax's denominator), or retention; the feed-forward a mixture of experts without gates beside a
shared one with a gate number a token. A layer may run with another's weights. Importing the package registers the
architecture."""
from .config import ZudusunConfig  # noqa: F401
from .spec import ARCHITECTURE, zudusun_spec  # noqa: F401
