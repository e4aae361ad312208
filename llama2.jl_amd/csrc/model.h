// The objects behind the handles of include/l2h.h, shared by the C-ABI layer (api.cpp) and the layered models
// (layered.cpp).
#pragma once

#include <algorithm>
#include <string>
#include <vector>

#include "l2h_internal.h"

struct l2h_ctx {
    int device = 0;
    hipStream_t stream = nullptr;
    std::string err;
    hipDeviceProp_t prop;
};

// records the message of a failed call on the context (or, without one, of a failed ctx_create) and returns `code`
int set_err(l2h_ctx *ctx, int code, const char *fmt, ...);

#define HIPCHK(ctx, call)                                                                          \
    do {                                                                                           \
        hipError_t e_ = (call);                                                                    \
        if (e_ != hipSuccess)                                                                      \
            return set_err((ctx), L2H_EHIP, "%s:%d: %s failed: %s", __FILE__, __LINE__, #call,     \
                           hipGetErrorString(e_));                                                 \
    } while (0)

static inline int64_t align256(int64_t v) { return (v + 255) & ~(int64_t)255; }

struct Layered;  // what a layered model adds (layered.cpp)

struct l2h_model {
    l2h_ctx *ctx = nullptr;
    l2h_config c{};
    int hs = 0, kv_dim = 0;
    float theta_scale = 0.0f;
    DevTensor glob[3];
    std::vector<DevTensor> layer;  // [n_layers][L2H_N_ROLES]
    bool finalized = false;
    // RunState (reference src/inference.jl:72-100) in device memory
    float *x = nullptr, *xb = nullptr, *xb2 = nullptr, *hb = nullptr, *hb2 = nullptr, *q = nullptr, *k = nullptr,
          *v = nullptr, *att = nullptr, *logits = nullptr;
    double *qd = nullptr, *pd = nullptr, *part = nullptr;
    float *rope_cs = nullptr;  // cos/sin of the current position's RoPE angles, [hs/2][2]
    float *kc = nullptr, *vc = nullptr;  // [n_layers] x per-layer cache
    int64_t cache_layer_elems = 0;
    DecodeCtl *ctl = nullptr;
    int32_t *prompt_dev = nullptr, *out_tokens = nullptr;
    int64_t *argmax_partial = nullptr;
    int max_out = 0;
    hipGraph_t graph = nullptr;
    hipGraphExec_t exec = nullptr;
    // persistent decode kernel
    int kv16 = 0;          // 1: the KV cache holds fp16 elements (l2h_model_set_kv_type)
    bool kv_uncached = false;       // the KV cache lives in uncached memory (see l2h_model_finalize)
    int flow_steps_per_launch = 1;  // steps of the token loop per launch of the streaming kernel
    int path_request = 0;  // 0 auto, 1 one kernel per phase, 2 persistent kernel, 3 streaming kernel (2, 3: required)
    bool mega = false;
    PhaseArgs mega_ph[5];  // q/k/v, wo, w1+w3, w2 of layer 0 and the classifier, planned for the persistent grid
    GridBar *bar = nullptr;
    unsigned long long bar_gen = 0;
    int mega_grid = 0;
    size_t mega_lds = 0;
    int mega_types[5] = {0, 0, 0, 0, 0};
#ifdef L2H_TIMELINE
    long long *timeline = nullptr, *timeline2 = nullptr;
#endif
    float *sample_p = nullptr;  // probabilities of the last l2h_sample call
    int32_t *sample_out = nullptr;
    // streaming decode kernel
    bool flow = false;
    FlowArgs flow_args{};
    int flow_grid = 0, flow_cls_type = 0;
    std::string flow_why;  // why the streaming kernel was not chosen (empty if it was, or if it was not asked for)
    unsigned int flow_gen = 1;  // epoch of the next launch's input; 0 is what cleared memory holds
    // batched prompt pass: buffers for pf_cap positions, allocated at the first l2h_prefill
    int pf_cap = 0;
    float *pf_x = nullptr, *pf_raw = nullptr, *pf_cs = nullptr;
    uint16_t *pf_xn = nullptr, *pf_q = nullptr, *pf_att = nullptr, *pf_hb = nullptr;
    int32_t *pf_tok = nullptr;
    unsigned char *pf_kvt = nullptr;  // one layer's K / V^T as bf16 tiles of 32 keys (k_pf_kv_tiles)
    int pf_kvt_tiles = 0;             // tiles per KV head
    // bf16 copy of the layer matrices for the prompt pass: per layer q|k|v rows, wo, w1/w3 rows in turn, w2
    int pf_copy_mode = 1;          // 0 never, 1 when it fits
    bool pf_copy_tried = false;
    uint16_t *pf_wbf = nullptr;
    // the plain products of the prompt pass (q | k | v, wo, w2) through hipBLASLt: asked for (default) / opened / the
    // layout the copy's three matrices have now (plain rows for the library, tiles for the own kernels)
    int pf_library_mode = 1;
    PfLt *pf_lt = nullptr;
    bool pf_lt_tried = false, pf_plain = false;
    std::string pf_lt_why, pf_lt_err;
    int64_t pf_wbf_layer = 0, pf_off_wo = 0, pf_off_w13 = 0, pf_off_w2 = 0;  // elements
    Layered *lay = nullptr;  // a model whose layers are described one by one (l2h_layered_create), else nullptr
    std::vector<void *> allocs;
    std::vector<void *> uc_allocs;  // blocks of the uncached pool (uncached_alloc), handed back with the model

    DevTensor &L(int layer_idx, int role) { return layer[(size_t)layer_idx * L2H_N_ROLES + role]; }
};

template <class T>
static int dalloc(l2h_model *m, T **p, int64_t n, bool zero) {
    void *v = nullptr;
    const size_t bytes = (size_t)std::max<int64_t>(n, 1) * sizeof(T);
    HIPCHK(m->ctx, hipMalloc(&v, bytes));
    m->allocs.push_back(v);
    if (zero) HIPCHK(m->ctx, hipMemset(v, 0, bytes));
    *p = (T *)v;
    return L2H_OK;
}

// ---- layered models (layered.cpp), as the C-ABI layer drives them ----------------------------------------------------
void layered_free(l2h_model *m);
int layered_set_tensor(l2h_model *m, int role, int layer, int expert, int type, const void *host, int64_t ne0, int64_t ne1);
int layered_finalize(l2h_model *m);             // checks the tensors, allocates the state and the decode buffers
int layered_reset(l2h_model *m);
int layered_check_pos(l2h_model *m, int pos0);  // may a call start at pos0?
void layered_advance(l2h_model *m, int pos);    // the state now holds positions 0 .. pos - 1
hipError_t layered_enqueue_token(l2h_model *m);  // embedding to logits
hipError_t layered_output(l2h_model *m);         // m->x -> m->logits
int layered_prefill_buffers(l2h_model *m, int cap, int n_want);
int layered_capacity(l2h_model *m);
bool layered_wants_library(l2h_model *m, int n);  // would a prompt of n positions run products through hipBLASLt?
int32_t *layered_token_buffer(l2h_model *m);
hipError_t layered_prefill_chunk(l2h_model *m, int M, int pos0);
int layered_prefill_logits(l2h_model *m, const int32_t *rows, int n, float *logits);
