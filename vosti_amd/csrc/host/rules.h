// Rules that every host of the kernels follows, written once: the native engine calls them directly, the
// Python package through the host library's C interface.  Two hosts that each computed them their own way
// could differ in a last bit (of a rotation frequency) or in a bucket's border, and with them the logits or
// the recorded graphs.
#pragma once
#include <cstdint>

namespace vosti {

// inv_freq[j] = 1 / theta^(2j / rotary_dim), j < rotary_dim / 2, as 32-bit values
// (python/vosti_kernels/rotary.py:80-90 writes 1.0 / (theta ** (arange(0, D, 2).float() / D)) in 32-bit).  The
// exponent is the 32-bit quotient; the power is the 32-bit number nearest to the exact power of the 32-bit
// theta and exponent (computed in 64-bit, then rounded once), so that it does not depend on whose powf runs;
// the reciprocal is a 32-bit division.
void rotary_inverse_frequencies(double theta, int rotary_dim, float* out);

// The frequencies of a rotation whose long wavelengths are stretched by `factor` so that positions beyond `original`
// stay inside the angles the model was trained on: with f[j] = theta^(-2j / rotary_dim) and
// turn(t) = rotary_dim * ln(original / (2 pi t)) / (2 ln theta), the pair whose wavelength makes t turns over `original`
// positions, lo = max(floor(turn(fast)), 0), hi = min(ceil(turn(slow)), rotary_dim - 1) and
// ramp[j] = clamp((j - lo) / max(hi - lo, 0.001), 0, 1), out[j] = f[j] / factor * ramp[j] + f[j] * (1 - ramp[j]),
// computed in 64-bit and rounded once.  Returns the factor on every cosine and sine, 0.1 ln(factor) + 1.
// factor <= 0: no stretch (out[j] = f[j], returns 1).
float rotary_stretched_frequencies(double theta, int rotary_dim, double factor, double original, double fast, double slow, float* out);

// The frequencies of a rotation whose positions are all stretched alike: out[j] = theta^(-2j / rotary_dim) / factor,
// computed in 64-bit and rounded once.  factor 1: the plain frequencies.
void rotary_linear_frequencies(double theta, int rotary_dim, double factor, float* out);

// The frequencies of a rotation that treats bands of wavelengths apart: with f[j] = theta^(-2j / rotary_dim) and its wavelength
// w = 2 pi / f[j], out[j] = f[j] for w < original / high, f[j] / factor for w > original / low, and between the two
// (1 - s) f[j] / factor + s f[j] with s = (original / w - low) / (high - low); computed in 64-bit and rounded once.
void rotary_banded_frequencies(double theta, int rotary_dim, double factor, double original, double low, double high, float* out);

// The class of a distance n >= 0 among `rows`: one each for the distances below rows / 2, then logarithmic ones,
// min(rows - 1, half + floor(ln(n / half) / ln(far / half) * (rows - half))) with half = rows / 2 (rounded down).
int distance_class(int64_t n, int64_t rows, double far);

// Recorded decode steps have one of 1, 2, 3, 4, 6, 8, 12, 16, 24, ... rows (a step with fewer is filled up with
// rows that read one key and store nothing; the reference pads its graphs likewise,
// python/vosti_kernels/graph_overlay.py:177-389), and block tables one of these numbers times eight pages, so
// that a long generation walks through few recordings.  More than 512 rows are recorded as they are.
int graph_row_bucket(int rows);
int graph_width_bucket(int pages);

// Recorded graphs kept; the least recently replayed one goes first.
constexpr int kMaxGraphs = 24;

}  // namespace vosti
