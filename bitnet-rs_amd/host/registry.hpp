// registry.hpp -- which model class serves a path.  A design with a folder (config.json + model.safetensors) registers the name
// its config.json carries in "architecture"; a single-file format registers its suffix.  Model files register themselves, so a
// program holds exactly the designs it was linked with.
#pragma once

#include <memory>
#include <string>
#include <vector>

#include "json.hpp"
#include "sequence.hpp"

namespace bitnet_host {

struct OpenOptions {
    bool f32 = false;   // every activation, cache and product in 32-bit (where the design has such a mode)
    int max_pos = 4096;  // positions a sequence may reach
};

using ArchitectureFactory = Sequence *(*)(const Json &config, const std::string &dir, const OpenOptions &opt, std::string &err);
using FileFactory = Sequence *(*)(const std::string &path, const OpenOptions &opt, std::string &err);

struct RegisterArchitecture {
    RegisterArchitecture(const char *name, ArchitectureFactory make);
};
struct RegisterFileFormat {
    RegisterFileFormat(const char *suffix, FileFactory make);
};
std::vector<std::string> registered_names();

// null + err on failure (unknown architecture, bad configuration, missing tensor, no device)
Sequence *open_model(const std::string &path, const OpenOptions &opt, std::string &err);

}  // namespace bitnet_host

// C shim: what every model shares.  Handles come from bitnet_host_open_model or bitnet_host_create.
extern "C" {
void *bitnet_host_open_model(const char *path, int f32, int max_pos);  // null: bitnet_host_open_error()
const char *bitnet_host_open_error(void);                              // thread-local
const char *bitnet_host_registered(void);                              // comma-separated names and suffixes
void bitnet_host_destroy(void *d);
const char *bitnet_host_error(void *d);
int bitnet_host_vocab(void *d);
int bitnet_host_width(void *d);
int bitnet_host_reset(void *d);
int bitnet_host_feed(void *d, const int32_t *tokens, int n);
int bitnet_host_run(void *d, int n, int with_logits, int use_graph, float *elapsed_ms);
int bitnet_host_prefill(void *d, int n, int with_logits, int digits, float *elapsed_ms);
// the next n tokens, forced; logits [n_want][vocab] of the places `want` among them
int bitnet_host_forward(void *d, const int32_t *tokens, int n, const int32_t *want, int n_want, float *logits);
int bitnet_host_prepare_graphs(void *d, int with_logits);
int bitnet_host_position(void *d);
int bitnet_host_history(void *d, int32_t *out, int n);
int bitnet_host_last_logits(void *d, float *out);
int bitnet_host_last_hidden(void *d, float *out);
uint64_t bitnet_host_weight_bytes(void *d);
}
