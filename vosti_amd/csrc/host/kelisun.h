// The Kelisun decoder, from its config.json to a description of parts: a normed embedding onto a residual of several streams
// in 32-bit that every sublayer reads and writes through learned coefficients, and layers listed one by one in the
// configuration: attention through a latent over a window of the last keys, one rotated key part for all heads with
// stretched frequencies, a learned sink per head; then a mixture of gated experts chosen by groups, weighted with their
// softmax scores as they are.  A layer may use an earlier or later layer's weights with a cache of its own.  Then the sum of
// the streams, the model's norm and an untied vocabulary projection.
#pragma once
#include "spec.h"

namespace vosti {

ModelSpec kelisun_model_spec(const Json& config);

}  // namespace vosti
