"""The Gubulorn design: post-norm layers (norms whose weight is stored around zero, a factor on the stream inside the
sum), the mixer either a gated delta rule or softmax attention (a norm a head, a temperature on late queries, a sink, a
gate a head) and a selective state space side by side, each result normed, the feed-forward dense with clamped
halves or a mixture of experts chosen inside groups, some of which hand their input through. Importing the package
registers the architecture."""
from .config import GubulornConfig  # noqa: F401
from .spec import ARCHITECTURE, gubulorn_spec  # noqa: F401
