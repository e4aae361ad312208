// Layered models: a decoder whose layers are described one by one (l2h_layered_create): which mixer (windowed attention, gated
// delta rule), which feed-forward (none, dense, mixture of experts), an optional per-token input per layer.  This file holds
// their tensors and per-sequence state and issues their launch sequences; the token loop, the recorded graph, argmax, sampling
// and the prompt pass's chunking are the library's own (api.cpp).
#include <math.h>
#include <string.h>

#include "layered.h"
#include "model.h"

namespace {
struct LayerDev {
    l2h_layer d{};
    uint64_t have = 0;  // bit per role that has been set
    LMat in;            // every row that reads the mixer's input: q | k | v | (gates) or q | k | v | beta | factors
    LMat o, a2, g2, up, down, router, side_gate, side_proj;
    std::vector<uint8_t> have_up, have_down;  // experts
    float *norm1 = nullptr, *norm2 = nullptr, *mixnorm = nullptr, *side_norm = nullptr, *conv = nullptr, *rate = nullptr,
          *bias = nullptr, *freq = nullptr;
    // per sequence
    float *kc = nullptr, *vc = nullptr;      // attention
    float *ring = nullptr, *state = nullptr;  // delta rule
};
}  // namespace

struct Layered {
    l2h_layered_config c{};
    std::vector<LayerDev> layer;
    LMat head;
    uint16_t *side_emb = nullptr;
    float *final_norm = nullptr;
    uint64_t have = 0;
    int pos = 0;  // positions the state has taken in
    // one token
    float *x_alt = nullptr, *in = nullptr, *mix = nullptr, *ssq = nullptr, *gate = nullptr, *hid = nullptr, *z = nullptr,
          *se = nullptr, *y = nullptr, *part = nullptr;
    // prompt pass, for `cap` positions
    int cap = 0;
    int32_t *tok = nullptr, *choice = nullptr, *slot_row = nullptr, *slot_of = nullptr, *n_tiles = nullptr, *want = nullptr;
    GemmTile *tiles = nullptr;
    float *X = nullptr, *raw = nullptr, *qkv = nullptr, *kq = nullptr, *beta = nullptr, *lg = nullptr, *gt = nullptr, *ob = nullptr,
          *zb = nullptr, *score = nullptr, *slot_scale = nullptr, *yb = nullptr, *Y = nullptr, *wl = nullptr, *rec = nullptr;
    void *xn = nullptr, *fa = nullptr, *fg = nullptr, *ao = nullptr, *hb = nullptr, *sb = nullptr;
    int want_cap = 0;
    // residual stream after every layer of the last prompt pass (l2h_layered_keep)
    bool keep = false;
    bool images_tried = false;
    unsigned char *kvt = nullptr;  // one attention layer's keys and values as the attention kernel's tiles
    float *kept = nullptr;
    int kept_cap = 0, kept_n = 0;

    int W() const { return c.width; }
    int ldw() const { return pad64(c.width); }
    int asize() const { return c.precision ? 4 : 2; }
};

static WindowShape window_shape(const Layered *l, const LayerDev &L) {
    WindowShape w{};
    w.H = L.d.n_heads, w.G = L.d.n_kv_heads, w.D = L.d.dim, w.V = L.d.vdim;
    w.window = L.d.window, w.rot = L.d.rot_dims, w.gated = L.d.head_gate, w.qk_norm = L.d.qk_norm;
    w.scale = L.d.scale, w.eps = l->c.norm_eps;
    w.seq_len = l->c.seq_len;
    return w;
}
static DeltaShape delta_shape(const Layered *l, const LayerDev &L) {
    DeltaShape d{};
    d.H = L.d.n_heads, d.G = L.d.n_kv_heads, d.D = L.d.dim, d.V = L.d.vdim;
    d.taps = L.d.taps, d.ra = L.d.decay_rank, d.rg = L.d.gate_rank;
    d.eps = l->c.norm_eps;
    return d;
}
static int mixer_rows(const Layered *l, const LayerDev &L) {
    return L.d.mixer == L2H_MIX_ATTENTION ? window_shape(l, L).n_in() : delta_shape(l, L).n_in();
}

// head size of the matrix-core attention kernel that holds this layer's heads (0: none does), and the tiles of 32 keys that a
// chunk of `cap` positions can see
static int attention_tile_size(const l2h_layer &d) {
    for (int hs : {32, 64, 96, 128})
        if (std::max((d.dim + 3) / 4 * 4, d.vdim) <= hs) return hs;
    return 0;
}
static int attention_tiles(const Layered *l, const LayerDev &L, int cap) {
    return (int)std::min<int64_t>(((int64_t)l->c.seq_len + 31) / 32, ((int64_t)L.d.window + cap) / 32 + 2);
}

static int mat_alloc(l2h_model *m, LMat *t, int64_t rows, int K) {
    t->rows = rows;
    t->K = K;
    t->ld = pad64(K);
    return dalloc(m, &t->w, rows * t->ld, true);
}

// ------------------------------------------------------------------------------------------
// creation
// ------------------------------------------------------------------------------------------
extern "C" int l2h_layered_create(l2h_ctx *ctx, const l2h_layered_config *cfg, const l2h_layer *layers, l2h_model **out) {
    if (!ctx || !cfg || !layers || !out) return set_err(ctx, L2H_EINVAL, "l2h_layered_create: NULL argument");
    *out = nullptr;
    const l2h_layered_config &c = *cfg;
    if (c.width < 1 || c.vocab_size < 1 || c.n_layers < 1 || c.seq_len < 1 || c.side_dim < 0)
        return set_err(ctx, L2H_EINVAL, "width, vocab_size, n_layers and seq_len must be positive");
    if (c.precision != 0 && c.precision != 1) return set_err(ctx, L2H_EINVAL, "precision must be 0 (bf16) or 1 (fp32)");
    if (!(c.norm_eps >= 0.0f)) return set_err(ctx, L2H_EINVAL, "norm_eps must not be negative");
    if (c.width > 32768) return set_err(ctx, L2H_EINVAL, "width %d is larger than 32768", c.width);
    for (int i = 0; i < c.n_layers; i++) {
        const l2h_layer &d = layers[i];
        if (d.mixer != L2H_MIX_ATTENTION && d.mixer != L2H_MIX_CHANNEL_DELTA) return set_err(ctx, L2H_EINVAL, "layer %d: unknown mixer %d", i, d.mixer);
        if (d.n_heads < 1 || d.n_kv_heads < 1 || d.n_heads % d.n_kv_heads != 0)
            return set_err(ctx, L2H_EINVAL, "layer %d: %d heads over %d key/value heads", i, d.n_heads, d.n_kv_heads);
        if (d.dim < 1 || d.dim > 256 || d.vdim < 1 || d.vdim > 256)
            return set_err(ctx, L2H_EINVAL, "layer %d: head sizes %d, %d (1 to 256 are built)", i, d.dim, d.vdim);
        if ((int64_t)d.n_heads * d.vdim > 32768) return set_err(ctx, L2H_EINVAL, "layer %d: heads x value size above 32768", i);
        if (d.mixer == L2H_MIX_ATTENTION) {
            if (d.window < 1 || std::min(d.window, c.seq_len) > 900000) return set_err(ctx, L2H_EINVAL, "layer %d: window %d", i, d.window);
            if (d.rot_dims < 0 || d.rot_dims > d.dim || d.rot_dims % 2) return set_err(ctx, L2H_EINVAL, "layer %d: %d rotated of %d dimensions", i, d.rot_dims, d.dim);
            if (d.rot_dims && !(d.rot_base > 0.0)) return set_err(ctx, L2H_EINVAL, "layer %d: rotation base must be positive", i);
            if (d.rot_original > 0.0 && (!(d.rot_factor > 0.0) || !(d.rot_low > 0.0) || !(d.rot_high > d.rot_low)))
                return set_err(ctx, L2H_EINVAL, "layer %d: frequency scaling needs factor > 0 and 0 < low < high", i);
        } else if (d.taps < 1 || d.taps > 64 || d.decay_rank < 1 || d.decay_rank > 4096 || d.gate_rank < 1 || d.gate_rank > 4096) {
            return set_err(ctx, L2H_EINVAL, "layer %d: taps %d, ranks %d, %d", i, d.taps, d.decay_rank, d.gate_rank);
        }
        if (d.ff != L2H_FF_NONE && d.ff != L2H_FF_DENSE && d.ff != L2H_FF_EXPERTS) return set_err(ctx, L2H_EINVAL, "layer %d: unknown feed-forward %d", i, d.ff);
        if (d.ff != L2H_FF_NONE && (d.ff_dim < 1 || d.ff_act < 0 || d.ff_act > 2)) return set_err(ctx, L2H_EINVAL, "layer %d: feed-forward of %d, activation %d", i, d.ff_dim, d.ff_act);
        if (d.ff == L2H_FF_DENSE && d.ff_dim > 36864) return set_err(ctx, L2H_EINVAL, "layer %d: feed-forward of %d is larger than 36864", i, d.ff_dim);
        if (d.ff == L2H_FF_EXPERTS && (d.n_experts < 1 || d.n_experts > 1024 || d.top < 1 || d.top > d.n_experts || d.top > 64 ||
                                       (int64_t)d.top * pad64(d.ff_dim) > 36864))
            return set_err(ctx, L2H_EINVAL, "layer %d: %d of %d experts of %d", i, d.top, d.n_experts, d.ff_dim);
    }
    HIPCHK(ctx, hipSetDevice(ctx->device));
    l2h_model *m = new l2h_model();
    Layered *l = new Layered();
    m->ctx = ctx;
    m->lay = l;
    m->c.dim = c.width;
    m->c.n_layers = c.n_layers;
    m->c.vocab_size = c.vocab_size;
    m->c.seq_len = c.seq_len;
    l->c = c;
    l->layer.resize((size_t)c.n_layers);
    int rc = L2H_OK;
#define A(call) \
    if (rc == L2H_OK) rc = (call)
    A(mat_alloc(m, &l->head, c.vocab_size, c.width));
    A(dalloc(m, &l->final_norm, c.width, true));
    if (c.side_dim) A(dalloc(m, &l->side_emb, (int64_t)c.vocab_size * c.n_layers * c.side_dim, true));
    DevTensor &e = m->glob[L2H_TOK_EMB];
    e.type = L2H_TYPE_BF16;
    e.ne0 = c.width;
    e.ne1 = c.vocab_size;
    uint16_t *emb = nullptr;
    A(dalloc(m, &emb, (int64_t)c.vocab_size * c.width, true));
    e.qs = (const uint8_t *)emb;
    for (int i = 0; i < c.n_layers && rc == L2H_OK; i++) {
        LayerDev &L = l->layer[(size_t)i];
        L.d = layers[i];
        const l2h_layer &d = L.d;
        const int HV = d.n_heads * d.vdim;
        A(mat_alloc(m, &L.in, mixer_rows(l, L), c.width));
        A(mat_alloc(m, &L.o, c.width, HV));
        A(dalloc(m, &L.norm1, c.width, true));
        if (d.mixer == L2H_MIX_ATTENTION) {
            std::vector<float> f((size_t)d.rot_dims / 2 + 1, 0.0f);
            for (int k = 0; k < d.rot_dims / 2; k++) {
                double v = pow(d.rot_base, -2.0 * k / d.rot_dims);
                if (d.rot_original > 0.0) {
                    const double wl = 2.0 * M_PI / v;
                    if (wl > d.rot_original / d.rot_low)
                        v /= d.rot_factor;
                    else if (wl >= d.rot_original / d.rot_high) {
                        const double s = (d.rot_original / wl - d.rot_low) / (d.rot_high - d.rot_low);
                        v = (1.0 - s) * v / d.rot_factor + s * v;
                    }
                }
                f[(size_t)k] = (float)v;
            }
            A(dalloc(m, &L.freq, (int64_t)f.size(), false));
            if (rc == L2H_OK && hipMemcpy(L.freq, f.data(), f.size() * 4, hipMemcpyHostToDevice) != hipSuccess)
                rc = set_err(ctx, L2H_EHIP, "uploading the rotation frequencies failed");
        } else {
            const DeltaShape s = delta_shape(l, L);
            A(mat_alloc(m, &L.a2, d.n_heads * d.dim, d.decay_rank));
            A(mat_alloc(m, &L.g2, HV, d.gate_rank));
            A(dalloc(m, &L.conv, (int64_t)s.channels() * d.taps, true));
            A(dalloc(m, &L.rate, d.n_heads, true));
            A(dalloc(m, &L.bias, d.n_heads * d.dim, true));
            A(dalloc(m, &L.mixnorm, d.vdim, true));
        }
        if (d.ff != L2H_FF_NONE) {
            const int64_t n = d.ff == L2H_FF_EXPERTS ? d.n_experts : 1;
            A(dalloc(m, &L.norm2, c.width, true));
            A(mat_alloc(m, &L.up, n * d.ff_dim, c.width));
            A(mat_alloc(m, &L.down, n * c.width, d.ff_dim));
            if (d.ff == L2H_FF_EXPERTS) {
                A(mat_alloc(m, &L.router, n, c.width));
                L.have_up.assign((size_t)n, 0);
                L.have_down.assign((size_t)n, 0);
            }
        }
        if (c.side_dim) {
            A(mat_alloc(m, &L.side_gate, c.side_dim, c.width));
            A(mat_alloc(m, &L.side_proj, c.width, c.side_dim));
            A(dalloc(m, &L.side_norm, c.width, true));
        }
    }
#undef A
    if (rc != L2H_OK) {
        l2h_model_destroy(m);
        return rc;
    }
    *out = m;
    return L2H_OK;
}

void layered_free(l2h_model *m) {
    delete m->lay;
    m->lay = nullptr;
}

// ------------------------------------------------------------------------------------------
// tensors
// ------------------------------------------------------------------------------------------
static const char *layered_role_name(int r) {
    static const char *n[] = {"token embedding", "final norm", "output", "norm 1", "norm 2", "q", "k", "v", "mixer output", "up", "down", "(w3)",
                              "head gate", "beta", "decay rate", "decay bias", "decay factor in", "decay factor out", "gate factor in",
                              "gate factor out", "mixer norm", "q convolution", "k convolution", "v convolution", "router", "expert up",
                              "expert down", "side embedding", "side gate", "side projection", "side norm"};
    return (r >= 0 && r < L2H_N_LAYERED_ROLES) ? n[r] : "?";
}

static float bf16_value(uint16_t b) {
    const uint32_t u = (uint32_t)b << 16;
    float f;
    memcpy(&f, &u, 4);
    return f;
}

// where a tensor goes: rows of a matrix, or an fp32 vector
struct LSlot {
    LMat *mat = nullptr;
    int64_t row0 = 0;
    float *vec = nullptr;
    uint16_t *flat = nullptr;  // bf16, unpadded
    int64_t e0 = 0, e1 = 0;
    bool exp = false;
    int64_t across = 0;  // a vector of e1 rows stored column by column, this many floats apart
};

static int layered_slot(l2h_model *m, int role, int layer, int expert, LSlot *s) {
    Layered *l = m->lay;
    const l2h_layered_config &c = l->c;
    LSlot &t = *s;
    auto mat = [&](LMat *x, int64_t row0, int64_t rows) {
        t.mat = x;
        t.row0 = row0;
        t.e0 = x->K;
        t.e1 = rows;
    };
    auto vec = [&](float *v, int64_t n, int64_t rows = 1) {
        t.vec = v;
        t.e0 = n;
        t.e1 = rows;
    };
    switch (role) {
    case L2H_TOK_EMB:
        t.flat = (uint16_t *)m->glob[L2H_TOK_EMB].qs;
        t.e0 = c.width, t.e1 = c.vocab_size;
        return L2H_OK;
    case L2H_OUTPUT: mat(&l->head, 0, c.vocab_size); return L2H_OK;
    case L2H_RMS_FINAL: vec(l->final_norm, c.width); return L2H_OK;
    case L2H_SIDE_EMB:
        if (!c.side_dim) break;
        t.flat = l->side_emb;
        t.e0 = (int64_t)c.n_layers * c.side_dim, t.e1 = c.vocab_size;
        return L2H_OK;
    }
    if (layer < 0 || layer >= c.n_layers) return set_err(m->ctx, L2H_EINVAL, "%s: layer %d out of range", layered_role_name(role), layer);
    LayerDev &L = l->layer[(size_t)layer];
    const l2h_layer &d = L.d;
    const int H = d.n_heads, G = d.n_kv_heads, D = d.dim, V = d.vdim;
    const bool att = d.mixer == L2H_MIX_ATTENTION;
    const DeltaShape ds = delta_shape(l, L);
    const WindowShape ws = window_shape(l, L);
    switch (role) {
    case L2H_RMS_ATT: vec(L.norm1, c.width); return L2H_OK;
    case L2H_RMS_FFN:
        if (d.ff == L2H_FF_NONE) break;
        vec(L.norm2, c.width);
        return L2H_OK;
    case L2H_WQ: mat(&L.in, 0, att ? H * D : G * D); return L2H_OK;
    case L2H_WK: mat(&L.in, att ? ws.off_k() : G * D, G * D); return L2H_OK;
    case L2H_WV: mat(&L.in, att ? ws.off_v() : 2 * G * D, att ? G * V : H * V); return L2H_OK;
    case L2H_WO: mat(&L.o, 0, c.width); return L2H_OK;
    case L2H_HEAD_GATE:
        if (!att || !d.head_gate) break;
        mat(&L.in, ws.off_g(), H);
        return L2H_OK;
    case L2H_W1:
        if (d.ff != L2H_FF_DENSE) break;
        mat(&L.up, 0, d.ff_dim);
        return L2H_OK;
    case L2H_W2:
        if (d.ff != L2H_FF_DENSE) break;
        mat(&L.down, 0, c.width);
        return L2H_OK;
    case L2H_ROUTER:
        if (d.ff != L2H_FF_EXPERTS) break;
        mat(&L.router, 0, d.n_experts);
        return L2H_OK;
    case L2H_EXPERT_UP:
    case L2H_EXPERT_DOWN:
        if (d.ff != L2H_FF_EXPERTS) break;
        if (expert < 0 || expert >= d.n_experts) return set_err(m->ctx, L2H_EINVAL, "expert %d out of range", expert);
        if (role == L2H_EXPERT_UP)
            mat(&L.up, (int64_t)expert * d.ff_dim, d.ff_dim);
        else
            mat(&L.down, (int64_t)expert * c.width, c.width);
        return L2H_OK;
    case L2H_SIDE_GATE:
        if (!c.side_dim) break;
        mat(&L.side_gate, 0, c.side_dim);
        return L2H_OK;
    case L2H_SIDE_PROJ:
        if (!c.side_dim) break;
        mat(&L.side_proj, 0, c.width);
        return L2H_OK;
    case L2H_SIDE_NORM:
        if (!c.side_dim) break;
        vec(L.side_norm, c.width);
        return L2H_OK;
    }
    if (!att) switch (role) {
        case L2H_BETA: mat(&L.in, ds.off_b(), H); return L2H_OK;
        case L2H_DECAY_IN: mat(&L.in, ds.off_a(), d.decay_rank); return L2H_OK;
        case L2H_GATE_IN: mat(&L.in, ds.off_g(), d.gate_rank); return L2H_OK;
        case L2H_DECAY_OUT: mat(&L.a2, 0, H * D); return L2H_OK;
        case L2H_GATE_OUT: mat(&L.g2, 0, H * V); return L2H_OK;
        case L2H_DECAY_RATE:
            vec(L.rate, H);
            t.exp = true;
            return L2H_OK;
        case L2H_DECAY_BIAS: vec(L.bias, H * D); return L2H_OK;
        case L2H_MIX_NORM: vec(L.mixnorm, V); return L2H_OK;
        case L2H_CONV_Q:
        case L2H_CONV_K:
        case L2H_CONV_V:
            vec(L.conv + (role - L2H_CONV_Q) * G * D, d.taps, role == L2H_CONV_V ? H * V : G * D);
            t.across = ds.channels();
            return L2H_OK;
        }
    return set_err(m->ctx, L2H_EINVAL, "layer %d has no tensor \"%s\"", layer, layered_role_name(role));
}

int layered_set_tensor(l2h_model *m, int role, int layer, int expert, int type, const void *host, int64_t ne0, int64_t ne1) {
    l2h_ctx *ctx = m->ctx;
    Layered *l = m->lay;
    if (m->finalized) return set_err(ctx, L2H_ESTATE, "model already finalized");
    if (role < 0 || role >= L2H_N_LAYERED_ROLES) return set_err(ctx, L2H_EINVAL, "role %d out of range", role);
    LSlot s;
    const int rc = layered_slot(m, role, layer, expert, &s);
    if (rc) return rc;
    if (ne0 != s.e0 || ne1 != s.e1)
        return set_err(ctx, L2H_EINVAL, "%s (layer %d): shape (%lld, %lld) does not match config (%lld, %lld)", layered_role_name(role), layer,
                       (long long)ne0, (long long)ne1, (long long)s.e0, (long long)s.e1);
    if (type != L2H_TYPE_BF16 && !(type == L2H_TYPE_F32 && s.vec))
        return set_err(ctx, L2H_ETYPE, "%s: tensor type %d (matrices are bf16, vectors bf16 or fp32)", layered_role_name(role), type);
    HIPCHK(ctx, hipSetDevice(ctx->device));
    if (s.vec) {
        std::vector<float> v((size_t)(ne0 * ne1));
        for (size_t i = 0; i < v.size(); i++) {
            v[i] = type == L2H_TYPE_F32 ? ((const float *)host)[i] : bf16_value(((const uint16_t *)host)[i]);
            if (s.exp) v[i] = (float)exp((double)v[i]);
        }
        if (s.across) {  // [channel][tap] -> [tap][channel]
            std::vector<float> w((size_t)ne1);
            for (int64_t k = 0; k < ne0; k++) {
                for (int64_t i = 0; i < ne1; i++) w[(size_t)i] = v[(size_t)(i * ne0 + k)];
                HIPCHK(ctx, hipMemcpy(s.vec + k * s.across, w.data(), w.size() * 4, hipMemcpyHostToDevice));
            }
        } else {
            HIPCHK(ctx, hipMemcpy(s.vec, v.data(), v.size() * 4, hipMemcpyHostToDevice));
        }
    } else if (s.flat) {
        HIPCHK(ctx, hipMemcpy(s.flat, host, (size_t)(ne0 * ne1) * 2, hipMemcpyHostToDevice));
    } else {
        HIPCHK(ctx, hipMemcpy2D(s.mat->w + s.row0 * s.mat->ld, (size_t)s.mat->ld * 2, host, (size_t)ne0 * 2, (size_t)ne0 * 2, (size_t)ne1,
                                hipMemcpyHostToDevice));
    }
    if (role == L2H_TOK_EMB || role == L2H_OUTPUT || role == L2H_RMS_FINAL || role == L2H_SIDE_EMB) {
        l->have |= (uint64_t)1 << role;
    } else {
        LayerDev &L = l->layer[(size_t)layer];
        L.have |= (uint64_t)1 << role;
        if (role == L2H_EXPERT_UP) L.have_up[(size_t)expert] = 1;
        if (role == L2H_EXPERT_DOWN) L.have_down[(size_t)expert] = 1;
    }
    return L2H_OK;
}

// ------------------------------------------------------------------------------------------
// state
// ------------------------------------------------------------------------------------------
int layered_finalize(l2h_model *m) {
    l2h_ctx *ctx = m->ctx;
    Layered *l = m->lay;
    const l2h_layered_config &c = l->c;
    int n_in = 1, hv = 1, hid = 1, ne = 1, ssq = 1;
    int64_t part = 1;
    auto missing = [&](uint64_t have, int role, int layer) -> int {
        if (have >> role & 1) return L2H_OK;
        return set_err(ctx, L2H_ESTATE, "missing tensor \"%s\"%s%s", layered_role_name(role), layer >= 0 ? " of layer " : "",
                       layer >= 0 ? std::to_string(layer).c_str() : "");
    };
    int rc;
    for (int r : {L2H_TOK_EMB, L2H_OUTPUT, L2H_RMS_FINAL})
        if ((rc = missing(l->have, r, -1))) return rc;
    if (c.side_dim && (rc = missing(l->have, L2H_SIDE_EMB, -1))) return rc;
#define DA(p, n, z)                       \
    if ((rc = dalloc(m, &(p), (n), (z)))) \
        return rc;
    for (int i = 0; i < c.n_layers; i++) {
        LayerDev &L = l->layer[(size_t)i];
        const l2h_layer &d = L.d;
        std::vector<int> need = {L2H_RMS_ATT, L2H_WQ, L2H_WK, L2H_WV, L2H_WO};
        if (d.mixer == L2H_MIX_ATTENTION) {
            if (d.head_gate) need.push_back(L2H_HEAD_GATE);
        } else {
            for (int r : {L2H_BETA, L2H_DECAY_RATE, L2H_DECAY_BIAS, L2H_DECAY_IN, L2H_DECAY_OUT, L2H_GATE_IN, L2H_GATE_OUT, L2H_MIX_NORM,
                          L2H_CONV_Q, L2H_CONV_K, L2H_CONV_V})
                need.push_back(r);
        }
        if (d.ff != L2H_FF_NONE) need.push_back(L2H_RMS_FFN);
        if (d.ff == L2H_FF_DENSE) need.push_back(L2H_W1), need.push_back(L2H_W2);
        if (d.ff == L2H_FF_EXPERTS) {
            need.push_back(L2H_ROUTER);
            for (int e = 0; e < d.n_experts; e++)
                if (!L.have_up[(size_t)e] || !L.have_down[(size_t)e]) return set_err(ctx, L2H_ESTATE, "missing expert %d of layer %d", e, i);
        }
        if (c.side_dim)
            for (int r : {L2H_SIDE_GATE, L2H_SIDE_PROJ, L2H_SIDE_NORM}) need.push_back(r);
        for (int r : need)
            if ((rc = missing(L.have, r, i))) return rc;
        if (d.mixer == L2H_MIX_ATTENTION) {
            const WindowShape w = window_shape(l, L);
            DA(L.kc, (int64_t)w.G * w.Dp() * w.seq_len, true);
            DA(L.vc, (int64_t)w.G * w.V * w.seq_len, true);
            part = std::max(part, window_part_floats(w));
        } else {
            const DeltaShape s = delta_shape(l, L);
            DA(L.ring, (int64_t)s.taps * s.channels(), true);
            DA(L.state, (int64_t)s.H * s.D * s.V, true);
            ssq = std::max(ssq, s.H * delta_splits(s.V));
        }
        n_in = std::max(n_in, mixer_rows(l, L));
        hv = std::max(hv, d.n_heads * d.vdim);
        if (d.ff != L2H_FF_NONE) hid = std::max(hid, d.ff_dim * (d.ff == L2H_FF_EXPERTS ? d.top : 1));
        if (d.ff == L2H_FF_EXPERTS) ne = std::max(ne, d.n_experts);
    }
    DA(m->x, c.width, true);
    DA(l->x_alt, c.width, true);
    DA(l->in, n_in, true);
    DA(l->mix, hv, true);
    DA(l->gate, hv, true);
    DA(l->ssq, ssq, true);
    DA(l->hid, hid, true);
    DA(l->z, ne, true);
    DA(l->se, std::max(1, c.side_dim), true);
    DA(l->y, c.width, true);
    DA(l->part, part, true);
    DA(m->rope_cs, 2, true);
    DA(m->logits, c.vocab_size, true);
#undef DA
    l->pos = 0;
    return L2H_OK;
}

// A sequence starts at position 0, where the kernels take the recurrent state as zero whatever it holds; from then on its
// positions come in order.
int layered_check_pos(l2h_model *m, int pos0) {
    Layered *l = m->lay;
    if (pos0 == 0 || pos0 == l->pos) return L2H_OK;
    return set_err(m->ctx, L2H_EINVAL, "position %d does not continue the sequence, whose state holds %d positions", pos0, l->pos);
}
void layered_advance(l2h_model *m, int pos) { m->lay->pos = pos; }

int layered_reset(l2h_model *m) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    for (LayerDev &L : l->layer) {
        const l2h_layer &d = L.d;
        if (d.mixer == L2H_MIX_ATTENTION) {
            const WindowShape w = window_shape(l, L);
            HIPCHK(m->ctx, hipMemsetAsync(L.kc, 0, (size_t)w.G * w.Dp() * w.seq_len * 4, s));
            HIPCHK(m->ctx, hipMemsetAsync(L.vc, 0, (size_t)w.G * w.V * w.seq_len * 4, s));
        } else {
            const DeltaShape t = delta_shape(l, L);
            HIPCHK(m->ctx, hipMemsetAsync(L.ring, 0, (size_t)t.taps * t.channels() * 4, s));
            HIPCHK(m->ctx, hipMemsetAsync(L.state, 0, (size_t)t.H * t.D * t.V * 4, s));
        }
    }
    HIPCHK(m->ctx, hipStreamSynchronize(s));
    l->pos = 0;
    return L2H_OK;
}

// ------------------------------------------------------------------------------------------
// one token
// ------------------------------------------------------------------------------------------
#define CK(call)                       \
    do {                               \
        e = (call);                    \
        if (e != hipSuccess) return e; \
    } while (0)

static RowsArgs rows_of(const LMat &w, const float *x, float *out) {
    RowsArgs a;
    a.w = w.w;
    a.ld = w.ld;
    a.K = w.K;
    a.n_rows = w.rows;
    a.x = x;
    a.out = out;
    return a;
}

// The residual stream moves to the other of its two buffers where a layer's pending per-token update is applied, by the
// launch that reads it next; it ends in m->x.
static float *stream_buf(const l2h_model *m, int layer) {
    const Layered *l = m->lay;
    return (l->c.side_dim && ((l->c.n_layers - layer) & 1)) ? l->x_alt : m->x;
}

// norm of the residual stream (with the update that the layer before left pending) and a matrix
static RowsArgs normed(const l2h_model *m, int layer, const LMat &w, const float *normw, float *out) {
    const Layered *l = m->lay;
    RowsArgs a = rows_of(w, stream_buf(m, layer), out);
    a.normw = normw;
    a.eps = l->c.norm_eps;
    if (l->c.side_dim && layer > 0) {
        a.x = stream_buf(m, layer - 1);
        a.y = l->y;
        a.yw = l->layer[(size_t)layer - 1].side_norm;
        a.mult = l->c.residual_mult;
        a.x_out = stream_buf(m, layer);
    }
    return a;
}

hipError_t layered_output(l2h_model *m) {
    Layered *l = m->lay;
    RowsArgs a = rows_of(l->head, m->x, m->logits);
    a.normw = l->final_norm;
    a.eps = l->c.norm_eps;
    return k_rows(m->ctx->stream, a, RP_NORM, RE_STORE, m->ctx->prop.multiProcessorCount);
}

hipError_t layered_enqueue_token(l2h_model *m) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const int cu = m->ctx->prop.multiProcessorCount;
    const l2h_layered_config &c = l->c;
    hipError_t e;
    CK(k_embed(s, m->glob[L2H_TOK_EMB], m->ctl, m->prompt_dev, stream_buf(m, 0), m->rope_cs, 0, 1.0f));
    for (int i = 0; i < c.n_layers; i++) {
        LayerDev &L = l->layer[(size_t)i];
        const l2h_layer &d = L.d;
        float *x = stream_buf(m, i);
        CK(k_rows(s, normed(m, i, L.in, L.norm1, l->in), RP_NORM, RE_STORE, cu));
        RowsArgs o = rows_of(L.o, l->mix, x);
        o.resid = x;
        o.mult = c.residual_mult;
        if (d.mixer == L2H_MIX_ATTENTION) {
            CK(k_window_step(s, window_shape(l, L), L.freq, l->in, L.kc, L.vc, m->ctl, l->part, l->mix));
            CK(k_rows(s, o, RP_PLAIN, RE_RESID, cu));
        } else {
            const DeltaWeights w = {L.conv, L.rate, L.bias, L.a2.w, L.g2.w, L.a2.ld, L.g2.ld};
            CK(k_delta_step(s, delta_shape(l, L), w, l->in, L.ring, L.state, m->ctl, l->mix, l->ssq, l->gate));
            o.normw = L.mixnorm;
            o.eps = c.norm_eps;
            o.ssq = l->ssq;
            o.gate = l->gate;
            o.hv = d.vdim;
            o.n_split = delta_splits(d.vdim);
            CK(k_rows(s, o, RP_HEADNORM, RE_RESID, cu));
        }
        if (d.ff != L2H_FF_NONE) {
            RowsArgs up = rows_of(L.up, x, l->hid), down = rows_of(L.down, l->hid, x);
            up.normw = L.norm2;
            up.eps = c.norm_eps;
            up.act = d.ff_act;
            down.resid = x;
            down.mult = c.residual_mult;
            if (d.ff == L2H_FF_DENSE) {
                CK(k_rows(s, up, RP_NORM, RE_ACT, cu));
                CK(k_rows(s, down, RP_PLAIN, RE_RESID, cu));
            } else {
                RowsArgs r = rows_of(L.router, x, l->z);
                r.normw = L.norm2;
                r.eps = c.norm_eps;
                CK(k_rows(s, r, RP_NORM, RE_STORE, cu));
                for (RowsArgs *a : {&up, &down}) {
                    a->z = l->z;
                    a->n_experts = d.n_experts;
                    a->top = d.top;
                }
                up.rows_each = d.ff_dim;
                up.n_rows = (int64_t)d.top * d.ff_dim;
                down.rows_each = c.width;
                down.n_rows = c.width;
                CK(k_rows(s, up, RP_UP, RE_UP, cu));
                CK(k_rows(s, down, RP_DOWN, RE_RESID, cu));
            }
        }
        if (c.side_dim) {
            RowsArgs g = rows_of(L.side_gate, x, l->se);
            g.act = LACT_GELU_TANH;
            g.emb = l->side_emb + (int64_t)i * c.side_dim;
            g.emb_ld = (int64_t)c.n_layers * c.side_dim;
            g.ctl = m->ctl;
            g.prompt = m->prompt_dev;
            CK(k_rows(s, g, RP_PLAIN, RE_EMBED, cu));
            CK(k_rows(s, rows_of(L.side_proj, l->se, l->y), RP_PLAIN, RE_STORE, cu));
        }
    }
    CK(k_rows(s, normed(m, c.n_layers, l->head, l->final_norm, m->logits), RP_NORM, RE_STORE, cu));
    return hipSuccess;
}

// ------------------------------------------------------------------------------------------
// prompt pass
// ------------------------------------------------------------------------------------------
// The matrices whose products have arithmetic behind them or are grouped (dense up, experts) get a second copy as tile images
// for the matrix-core kernel of the prompt pass, made once, where it fits beside 2 GiB of free memory.
#define L_IMAGE_MIN_ROWS 192  // a row group of an image is 256 rows: smaller matrices stay with k_gemm
#define L_BIG_MIN_M 128       // positions from which the library and the images are used
static int prompt_images(l2h_model *m) {
    Layered *l = m->lay;
    if (l->images_tried || l->c.precision || !m->pf_copy_mode) return L2H_OK;
    l->images_tried = true;
    struct Job {
        LMat *w;
        int64_t rows, n;
    };
    std::vector<Job> jobs;
    int64_t elems = 0;
    auto add = [&](LMat *w, int64_t rows, int64_t n) {
        if (rows < L_IMAGE_MIN_ROWS) return;
        jobs.push_back(Job{w, rows, n});
        elems += n * k_tile_image_elems(rows, w->ld);
    };
    for (LayerDev &L : l->layer) {
        if (L.d.ff == L2H_FF_DENSE) add(&L.up, L.d.ff_dim, 1);
        if (L.d.ff == L2H_FF_EXPERTS) {
            if (std::min(L.d.ff_dim, l->W()) < L_IMAGE_MIN_ROWS) continue;  // (both or neither)
            add(&L.up, L.d.ff_dim, L.d.n_experts);
            add(&L.down, l->W(), L.d.n_experts);
        }
    }
    size_t free_b = 0, total_b = 0;
    HIPCHK(m->ctx, hipMemGetInfo(&free_b, &total_b));
    if (free_b < (size_t)elems * 2 + ((size_t)2 << 30)) return L2H_OK;
    for (const Job &j : jobs) {
        uint16_t *p = nullptr;
        const int rc = dalloc(m, &p, j.n * k_tile_image_elems(j.rows, j.w->ld), false);
        if (rc) return rc;
        HIPCHK(m->ctx, k_tile_image(m->ctx->stream, j.w->w, j.w->ld, j.rows, j.n, p));
        j.w->image = p;
        j.w->image_stride = k_tile_image_elems(j.rows, j.w->ld);
    }
    HIPCHK(m->ctx, hipStreamSynchronize(m->ctx->stream));
    return L2H_OK;
}

int layered_prefill_buffers(l2h_model *m, int cap, int n_want) {
    Layered *l = m->lay;
    const l2h_layered_config &c = l->c;
    int rc;
    cap = (cap + 255) / 256 * 256;  // (a library product computes whole groups of 128 positions)
    if (cap > L_BIG_MIN_M && (rc = prompt_images(m))) return rc;
#define DA(p, n)                            \
    if ((rc = dalloc(m, &(p), (n), false))) \
        return rc;
#define DB(p, n)                                      \
    {                                                 \
        char *b_ = nullptr;                           \
        DA(b_, (int64_t)(n) * l->asize())             \
        (p) = b_;                                     \
    }
    if (n_want > l->want_cap) {
        DA(l->want, n_want);
        DA(l->wl, (int64_t)((n_want + 255) / 256 * 256) * c.vocab_size);
        l->want_cap = n_want;
    }
    if (l->keep && l->kept_cap < cap) {
        DA(l->kept, (int64_t)c.n_layers * cap * c.width);
        l->kept_cap = cap;
    }
    if (l->cap >= cap) return L2H_OK;
    int64_t n_in = 1, ch = 1, g = 1, h = 1, hd = 1, hv = 1, lhv = 64, lra = 64, lrg = 64, hid = 64, ne = 1, slots = 1, up_slots = 1, tiles = 1;
    int64_t kvt = 0, rec = 0;
    bool moe = false;
    for (LayerDev &L : l->layer) {
        const l2h_layer &d = L.d;
        n_in = std::max<int64_t>(n_in, mixer_rows(l, L));
        hv = std::max<int64_t>(hv, d.n_heads * d.vdim);
        lhv = std::max<int64_t>(lhv, L.o.ld);
        if (d.mixer == L2H_MIX_ATTENTION) {
            ch = std::max<int64_t>(ch, d.n_heads * d.dim);
            const int hs = attention_tile_size(d);
            if (hs && !c.precision) {
                ch = std::max<int64_t>(ch, d.n_heads * hs);
                kvt = std::max<int64_t>(kvt, (int64_t)d.n_kv_heads * attention_tiles(l, L, cap) * k_pf_kv_tile_bytes(hs));
            }
        } else {
            ch = std::max<int64_t>(ch, delta_shape(l, L).channels());
            g = std::max<int64_t>(g, d.n_kv_heads);
            h = std::max<int64_t>(h, d.n_heads);
            hd = std::max<int64_t>(hd, d.n_heads * d.dim);
            lra = std::max<int64_t>(lra, L.a2.ld);
            rec = std::max(rec, delta_walk_floats(delta_shape(l, L), cap));
            lrg = std::max<int64_t>(lrg, L.g2.ld);
        }
        if (d.ff == L2H_FF_DENSE) hid = std::max<int64_t>(hid, L.down.ld);
        if (d.ff == L2H_FF_EXPERTS) {
            moe = true;
            ne = std::max<int64_t>(ne, d.n_experts);
            slots = std::max<int64_t>(slots, d.top);
            up_slots = std::max<int64_t>(up_slots, (int64_t)d.top * L.down.ld);
            tiles = std::max<int64_t>(tiles, ((int64_t)cap * d.top + L_GEMM_TILE - 1) / L_GEMM_TILE + d.n_experts);
        }
    }
    if (kvt) DA(l->kvt, kvt);
    if (rec) DA(l->rec, rec);
    DA(l->tok, cap);
    DA(l->X, (int64_t)cap * c.width);
    DA(l->raw, cap * std::max<int64_t>(n_in, c.side_dim));
    DA(l->qkv, cap * ch);
    DA(l->kq, cap * g);
    DA(l->beta, cap * h);
    DA(l->lg, cap * hd);
    DA(l->gt, cap * hv);
    DA(l->ob, cap * hv);
    DB(l->xn, (int64_t)cap * l->ldw());
    DB(l->fa, cap * lra);
    DB(l->fg, cap * lrg);
    DB(l->ao, cap * lhv);
    DB(l->hb, cap * std::max(hid, moe ? up_slots : (int64_t)0));
    if (moe) {
        DA(l->zb, cap * ne);
        DA(l->choice, cap * slots);
        DA(l->score, cap * slots);
        DA(l->slot_row, cap * slots);
        DA(l->slot_scale, cap * slots);
        DA(l->slot_of, cap * slots);
        DA(l->tiles, tiles);
        DA(l->n_tiles, 1);
        DA(l->yb, cap * slots * c.width);
    }
    if (c.side_dim) {
        DB(l->sb, (int64_t)cap * pad64(c.side_dim));
        DA(l->Y, (int64_t)cap * c.width);
    }
#undef DB
#undef DA
    l->cap = cap;
    return L2H_OK;
}
bool layered_wants_library(l2h_model *m, int n) {
    const Layered *l = m->lay;
    return l->c.precision == 0 && n >= L_BIG_MIN_M && (double)n * l->ldw() * l->layer[0].in.rows >= (double)(1 << 28);
}
int32_t *layered_token_buffer(l2h_model *m) { return m->lay->tok; }
int layered_capacity(l2h_model *m) { return m->lay->cap; }

static GemmArgs gemm_of(const LMat &w, const void *x, int M) {
    GemmArgs a;
    a.w = w.w;
    a.n_rows = w.rows;
    a.ld = w.ld;
    a.x = x;
    a.ldx = w.ld;
    a.M = M;
    return a;
}

// a product whose result stays fp32; large plain ones (GE_STORE, GE_RESID) go through the library, rounded up to whole groups of 128 positions so
// that few different shapes occur: the rows beyond M are computed from whatever the buffers hold, and never read
static bool library_takes(const l2h_model *m, const GemmArgs &a) {
    return m->lay->c.precision == 0 && m->pf_lt && m->pf_library_mode && a.M >= L_BIG_MIN_M &&
           (double)a.M * (double)a.n_rows * (double)a.ld >= (double)(1 << 26);
}
static hipError_t product(l2h_model *m, GemmArgs a, int epi, float *out, int64_t ldo, float mult) {
    if ((epi == GE_STORE || epi == GE_RESID) && library_takes(m, a)) {
        const int M = (a.M + 127) / 128 * 128;
        const hipError_t e = pf_lt_gemm(m->pf_lt, m->ctx->stream, a.w, (const uint16_t *)a.x, out, M, a.n_rows, a.ld, ldo, epi == GE_RESID,
                                        &m->pf_lt_err, mult);
        if (e != hipErrorNotSupported) return e;
        pf_lt_close(m->pf_lt);  // no algorithm for a shape: this library's own kernels from here on
        m->pf_lt = nullptr;
        (void)hipGetLastError();
    }
    a.outf = out;
    a.ldo = ldo;
    a.mult = mult;
    return k_gemm(m->ctx->stream, a, m->lay->c.precision, epi);
}
static bool image_takes(const LMat &w, int M) { return w.image && M >= L_BIG_MIN_M; }
static hipError_t to_acts(l2h_model *m, GemmArgs a, int epi, void *out, int64_t lda, const LMat *w = nullptr) {
    a.outa = out;
    a.lda = lda;
    if (w && image_takes(*w, a.M)) {
        a.w = w->image;
        return k_tiles(m->ctx->stream, a, epi);
    }
    return k_gemm(m->ctx->stream, a, m->lay->c.precision, epi);
}

static hipError_t prompt_delta(l2h_model *m, LayerDev &L, int M, int pos0) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const int prec = l->c.precision;
    const DeltaShape d = delta_shape(l, L);
    const int64_t ldr = d.n_in(), hd = d.H * d.D, hv = d.H * d.V;
    hipError_t e;
    CK(k_delta_prepare(s, d, L.conv, l->raw, ldr, L.ring, M, pos0, l->qkv, l->kq, l->beta, l->fa, L.a2.ld, l->fg, L.g2.ld, prec));
    CK(k_delta_ring(s, d, l->raw, ldr, L.ring, M, pos0));
    GemmArgs a = gemm_of(L.a2, l->fa, M);
    a.outf = l->lg;
    a.ldo = hd;
    a.rate = L.rate;
    a.bias = L.bias;
    a.hd = d.D;
    CK(k_gemm(s, a, prec, GE_DECAY));
    CK(product(m, gemm_of(L.g2, l->fg, M), GE_SIGMOID, l->gt, hv, 1.0f));
    if (M >= L_DELTA_WALK_MIN)
        CK(k_delta_walk(s, d, l->qkv, l->beta, l->lg, L.state, M, pos0, l->rec, l->ob));
    else
        CK(k_delta_scan(s, d, l->qkv, l->kq, l->beta, l->lg, L.state, M, pos0, l->ob));
    CK(k_head_norm_rows(s, l->ob, l->gt, L.mixnorm, M, d.H, d.V, d.eps, l->ao, L.o.ld, prec));
    return hipSuccess;
}

static hipError_t prompt_attention(l2h_model *m, LayerDev &L, int M, int pos0) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const WindowShape w = window_shape(l, L);
    const int64_t ldr = w.n_in();
    const int hs = attention_tile_size(L.d);
    hipError_t e;
    if (hs && l->c.precision == 0) {
        uint16_t *qb = (uint16_t *)l->qkv;
        PfWindow win;
        win.window = w.window;
        win.tile0 = std::max(0, pos0 - w.window + 1) / 32;
        win.vdim = w.V;
        win.scale = w.scale;
        win.gate = w.gated ? l->raw + w.off_g() : nullptr;
        win.ldg = ldr;
        win.ldo = L.o.ld;
        const int n_tiles = (pos0 + M + 31) / 32 - win.tile0, cap = attention_tiles(l, L, l->cap);
        CK(k_window_prepare(s, w, L.freq, l->raw, ldr, L.kc, L.vc, M, pos0, nullptr, qb, hs));
        CK(k_pf_kv_tiles(s, L.kc, L.vc, l->kvt, n_tiles, cap, hs, w.G, w.seq_len, win.tile0, w.Dp(), w.V));
        return k_pf_attention(s, qb, (uint16_t *)l->ao, l->kvt, cap, M, pos0, hs, w.H, w.G, w.H * hs, &win);
    }
    CK(k_window_prepare(s, w, L.freq, l->raw, ldr, L.kc, L.vc, M, pos0, l->qkv, nullptr, 0));
    CK(k_window_rows(s, w, l->qkv, l->raw, ldr, L.kc, L.vc, M, pos0, l->ao, L.o.ld, l->c.precision));
    return hipSuccess;
}

static hipError_t prompt_experts(l2h_model *m, LayerDev &L, int M) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const l2h_layer &d = L.d;
    const int prec = l->c.precision;
    hipError_t e;
    CK(product(m, gemm_of(L.router, l->xn, M), GE_STORE, l->zb, d.n_experts, 1.0f));
    CK(k_route(s, l->zb, M, d.n_experts, d.top, l->choice, l->score));
    const bool image = image_takes(L.up, M) && image_takes(L.down, M);
    const int rows = image ? L_IMAGE_TILE : L_GEMM_TILE;
    CK(k_group(s, l->choice, l->score, M, d.n_experts, d.top, l->slot_row, l->slot_scale, l->slot_of, l->tiles, l->n_tiles, rows));
    const int slots = M * d.top, max_tiles = (slots + rows - 1) / rows + d.n_experts;
    GemmArgs up = gemm_of(L.up, l->xn, slots), down = gemm_of(L.down, l->hb, slots);
    for (GemmArgs *a : {&up, &down}) {
        a->tiles = l->tiles;
        a->n_tiles = l->n_tiles;
        a->max_tiles = max_tiles;
    }
    up.n_rows = d.ff_dim;
    up.expert_stride = (int64_t)d.ff_dim * L.up.ld;
    up.gather = l->slot_row;
    up.row_scale = l->slot_scale;
    up.act = d.ff_act;
    up.outa = l->hb;
    up.lda = L.down.ld;
    if (image) {
        up.w = L.up.image;
        up.expert_stride = L.up.image_stride;
        CK(k_tiles(s, up, GE_UP));
    } else {
        CK(k_gemm(s, up, prec, GE_UP));
    }
    down.n_rows = l->W();
    down.expert_stride = (int64_t)l->W() * L.down.ld;
    down.outf = l->yb;
    down.ldo = l->W();
    if (image) {
        down.w = L.down.image;
        down.expert_stride = L.down.image_stride;
        CK(k_tiles(s, down, GE_STORE));
    } else {
        CK(k_gemm(s, down, prec, GE_STORE));
    }
    return k_gather_add(s, l->X, l->yb, l->slot_of, M, d.top, l->W(), l->c.residual_mult);
}

hipError_t layered_prefill_chunk(l2h_model *m, int M, int pos0) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const l2h_layered_config &c = l->c;
    const int W = c.width, ldw = l->ldw(), prec = c.precision;
    const float mult = c.residual_mult, eps = c.norm_eps;
    hipError_t e;
    CK(k_pf_embed(s, m->glob[L2H_TOK_EMB], l->tok, l->X, M));
    const float *py = nullptr, *pyw = nullptr;  // per-token update that waits for the next reader of the residual stream
    auto keep = [&](int layer) -> hipError_t {
        if (!l->keep || layer < 0) return hipSuccess;
        return hipMemcpyAsync(l->kept + ((int64_t)layer * l->kept_cap) * W, l->X, (size_t)M * W * 4, hipMemcpyDeviceToDevice, s);
    };
    for (int i = 0; i < c.n_layers; i++) {
        LayerDev &L = l->layer[(size_t)i];
        const l2h_layer &d = L.d;
        CK(k_norm_rows(s, l->X, W, M, L.norm1, eps, py, pyw, mult, nullptr, l->xn, ldw, prec));
        CK(keep(i - 1));
        CK(product(m, gemm_of(L.in, l->xn, M), GE_STORE, l->raw, L.in.rows, 1.0f));
        CK(d.mixer == L2H_MIX_ATTENTION ? prompt_attention(m, L, M, pos0) : prompt_delta(m, L, M, pos0));
        CK(product(m, gemm_of(L.o, l->ao, M), GE_RESID, l->X, W, mult));
        if (d.ff != L2H_FF_NONE) {
            CK(k_norm_rows(s, l->X, W, M, L.norm2, eps, nullptr, nullptr, mult, nullptr, l->xn, ldw, prec));
            if (d.ff == L2H_FF_DENSE) {
                GemmArgs up = gemm_of(L.up, l->xn, M);
                up.act = d.ff_act;
                CK(to_acts(m, up, GE_ACT, l->hb, L.down.ld, &L.up));
                CK(product(m, gemm_of(L.down, l->hb, M), GE_RESID, l->X, W, mult));
            } else {
                CK(prompt_experts(m, L, M));
            }
        }
        if (c.side_dim) {
            CK(k_norm_rows(s, l->X, W, M, nullptr, eps, nullptr, nullptr, mult, nullptr, l->xn, ldw, prec));
            GemmArgs g = gemm_of(L.side_gate, l->xn, M);
            g.act = LACT_GELU_TANH;
            g.emb = l->side_emb + (int64_t)i * c.side_dim;
            g.emb_ld = (int64_t)c.n_layers * c.side_dim;
            g.tokens = l->tok;
            if (library_takes(m, g)) {
                CK(product(m, g, GE_STORE, l->raw, c.side_dim, 1.0f));
                CK(k_embed_rows(s, l->raw, M, c.side_dim, g.act, g.emb, g.emb_ld, g.tokens, l->sb, L.side_proj.ld, prec));
            } else {
                CK(to_acts(m, g, GE_EMBED, l->sb, L.side_proj.ld));
            }
            CK(product(m, gemm_of(L.side_proj, l->sb, M), GE_STORE, l->Y, W, 1.0f));
            py = l->Y;
            pyw = L.side_norm;
        }
    }
    if (py) CK(k_norm_rows(s, l->X, W, M, nullptr, eps, py, pyw, mult, nullptr, nullptr, 0, prec));
    CK(keep(c.n_layers - 1));
    l->kept_n = M;
    // the last position becomes the decode state's residual stream
    return hipMemcpyAsync(m->x, l->X + (int64_t)(M - 1) * W, (size_t)W * 4, hipMemcpyDeviceToDevice, s);
}

// logits of n rows of the chunk just computed; rows[] (host) index the chunk's positions
int layered_prefill_logits(l2h_model *m, const int32_t *rows, int n, float *logits) {
    Layered *l = m->lay;
    l2h_ctx *ctx = m->ctx;
    const l2h_layered_config &c = l->c;
    HIPCHK(ctx, hipMemcpyAsync(l->want, rows, (size_t)n * 4, hipMemcpyHostToDevice, ctx->stream));
    for (int i = 0; i < n; i += l->cap) {  // (xn holds `cap` rows)
        const int k = std::min(l->cap, n - i);
        HIPCHK(ctx, k_norm_rows(ctx->stream, l->X, c.width, k, l->final_norm, c.norm_eps, nullptr, nullptr, 1.0f, l->want + i, l->xn, l->ldw(), c.precision));
        HIPCHK(ctx, product(m, gemm_of(l->head, l->xn, k), GE_STORE, l->wl + (int64_t)i * c.vocab_size, c.vocab_size, 1.0f));
    }
    HIPCHK(ctx, hipMemcpyAsync(logits, l->wl, (size_t)n * c.vocab_size * 4, hipMemcpyDeviceToHost, ctx->stream));
    HIPCHK(ctx, hipStreamSynchronize(ctx->stream));  // (rows and the buffers may be reused by the caller)
    return L2H_OK;
}

extern "C" int l2h_layered_keep(l2h_model *m, int on) {
    if (!m || !m->lay) return L2H_EINVAL;
    m->lay->keep = on != 0;
    return L2H_OK;
}
extern "C" int l2h_layered_kept(l2h_model *m, int layer, float *host, int64_t n) {
    if (!m || !m->lay || !host) return L2H_EINVAL;
    Layered *l = m->lay;
    if (!l->kept || layer < 0 || layer >= l->c.n_layers || n != (int64_t)l->kept_n * l->c.width)
        return set_err(m->ctx, L2H_EINVAL, "kept residual stream: layer %d, %lld floats (holds %d positions)", layer, (long long)n, l->kept_n);
    HIPCHK(m->ctx, hipStreamSynchronize(m->ctx->stream));
    HIPCHK(m->ctx, hipMemcpy(host, l->kept + (int64_t)layer * l->kept_cap * l->c.width, (size_t)n * 4, hipMemcpyDeviceToHost));
    return L2H_OK;
}
