// pybind11 module of the decoder subset (ops/build.py build("decoder")): the
// kernels a paged decoder model runs, for a first use without the full build.
#include "bindings_decoder.h"

PYBIND11_MODULE(_dnn_decoder, m) {
  m.doc() = "distributed_neural_networks_amd HIP/CDNA4 decoder kernels (gfx950)";
  m.attr("arch") = "gfx950";
  bind_decoder(m);
}
