// The Puvirax decoder, from its config.json to a description of parts: a token's embedding plus a row of a second table that
// the token and the one before it pick, a residual stream in 32-bit with a norm before every sublayer, and layers listed one
// by one in the configuration: softmax attention in three kinds (rotated with frequencies by bands, unit heads and a gate a
// head; windowed with head norms and a learned bias by distance; unwindowed with one norm over all heads and such a bias),
// whose values may be blended with the first such layer's; then a dense squared-relu layer, or experts chosen by groups with
// corrected logistic scores beside a shared expert.  The logits come from the embedding table, times a constant.
#pragma once
#include "spec.h"

namespace vosti {

ModelSpec puvirax_model_spec(const Json& config);

}  // namespace vosti
