// bamd_arch.cpp — the architectures this library loads
#include "bamd_arch.h"
#include "bamd_json.h"
#include "bamd_stack.h"
#include <sys/stat.h>
#include <fstream>
#include <iterator>

static const bamd_stack_design TUPITAR = [] {
    bamd_stack_design d = {};
    d.scaled_embedding = d.learned_positions = d.token_shift = true; d.norm = STACK_NORM_OUTPUT_SCALAR; d.mlp_act = STACK_ACT_POLYNORM;
    d.mixers = "mamba2 latent_attention"; d.latent_sink = d.latent_gate = true;
    return d;
}();
static const bamd_stack_design MAFURAX = [] {
    bamd_stack_design d = {};
    d.norm = STACK_NORM_SANDWICH; d.mlp_act = STACK_ACT_CLAMPED_GLU; d.tied_head = true;
    d.mixers = "parallel"; d.kv_unit = d.kv_cap = d.kv_bias = d.kv_gate = d.gla_gate = true;
    return d;
}();

static const bamd_arch TABLE[] = {
    { "llama", false, bamd_llama_load, nullptr },
    { "Tupitar", true, bamd_stack_load, &TUPITAR },
    { "Mafurax", true, bamd_stack_load, &MAFURAX },
};

const bamd_arch * bamd_arch_find(const std::string & name, bool folder) {
    for (const bamd_arch & a : TABLE) if (a.folder == folder && name == a.name) return &a;
    return nullptr;
}
std::string bamd_arch_names(bool folder) {
    std::string s;
    for (const bamd_arch & a : TABLE) if (a.folder == folder) s += (s.empty() ? "\"" : ", \"") + std::string(a.name) + "\"";
    return s;
}
bool bamd_is_folder(const std::string & path) { struct stat st; return stat(path.c_str(), &st) == 0 && S_ISDIR(st.st_mode); }
bool bamd_arch_of_folder(const std::string & path, std::string & name, std::string & err) {
    std::ifstream f(path + "/config.json", std::ios::binary);
    if (!f) { err = "cannot open " + path + "/config.json"; return false; }
    const std::string text((std::istreambuf_iterator<char>(f)), std::istreambuf_iterator<char>());
    Json j;
    if (!Json::parse(text.data(), text.data() + text.size(), j, err)) { err = path + "/config.json: " + err; return false; }
    const Json * a = j.get("architecture");
    if (!a || a->kind != Json::STR) { err = path + "/config.json: no \"architecture\""; return false; }
    name = a->str;
    return true;
}
