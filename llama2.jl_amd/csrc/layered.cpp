// Layered models: a decoder whose layers are described one by one (l2h_layered_create): which mixer (windowed attention, gated
// delta rule, latent attention), which feed-forward (none, dense, mixture of experts), one norm or two, an optional per-token
// input per layer; a stretch of layers may run several times over.  This file holds their tensors and per-sequence state and
// issues their launch sequences; the token loop, the recorded graph, argmax, sampling
// and the prompt pass's chunking are the library's own (api.cpp).
#include <math.h>
#include <string.h>

#include "layered.h"
#include "model.h"

namespace {
struct LayerDev {
    l2h_layer d{};
    uint64_t have = 0;  // bit per role that has been set
    // every row that reads the mixer's input: q | k | v | (gates) or q | k | v | beta | factors or what LatentShape says; in a
    // parallel layer also the router's rows and behind them (from row n_plain on) a gated dense feed-forward's.  up, down and
    // router then name parts of `in` and `o`.
    LMat in;
    int n_plain = 0, off_z = 0;
    // o: the mixer's output matrix; with `joined` its rows go on, at column o_cols, as the dense feed-forward's output matrix
    LMat o;
    bool joined = false;
    int o_cols = 0;
    LMat a2, g2, up, down, router, side_gate, side_proj, uq, ukv;
    std::vector<uint8_t> have_up, have_down, have_gate;  // experts
    float *norm1 = nullptr, *norm2 = nullptr, *mixnorm = nullptr, *side_norm = nullptr, *conv = nullptr, *rate = nullptr,
          *bias = nullptr, *freq = nullptr, *qnorm = nullptr, *kvnorm = nullptr, *router_bias = nullptr;
    bool stacked() const { return d.parallel && d.ff == L2H_FF_DENSE && d.ff_gated; }  // its feed-forward's rows are in `in`
    int up_rows() const { return d.ff_dim * (d.ff_gated ? 2 : 1); }                     // rows of up, of one expert's up
};
// One run of a layer: a looped layer has one for each pass.  What a sequence carries belongs to the run.
struct LayerRun {
    int layer = 0, pass = -1;                 // pass: of which this is the first layer (-1: of none)
    float *kc = nullptr, *vc = nullptr;       // attention; latent attention has its rows in kc
    float *ring = nullptr, *state = nullptr;  // delta rule
};
}  // namespace

struct Layered {
    l2h_layered_config c{};
    std::vector<LayerDev> layer;
    std::vector<LayerRun> run;
    LMat head;
    float *loop_step = nullptr;
    uint16_t *side_emb = nullptr;
    float *final_norm = nullptr;
    uint64_t have = 0;
    int pos = 0;  // positions the state has taken in
    // one token
    float *x_alt = nullptr, *in = nullptr, *mix = nullptr, *ssq = nullptr, *gate = nullptr, *hid = nullptr, *z = nullptr,
          *se = nullptr, *y = nullptr, *part = nullptr, *x0 = nullptr, *lq = nullptr, *qa = nullptr;
    // prompt pass, for `cap` positions
    int cap = 0;
    int32_t *tok = nullptr, *choice = nullptr, *slot_row = nullptr, *slot_of = nullptr, *n_tiles = nullptr, *want = nullptr;
    GemmTile *tiles = nullptr;
    float *X = nullptr, *raw = nullptr, *qkv = nullptr, *kq = nullptr, *beta = nullptr, *lg = nullptr, *gt = nullptr, *ob = nullptr,
          *zb = nullptr, *score = nullptr, *slot_scale = nullptr, *yb = nullptr, *Y = nullptr, *wl = nullptr, *rec = nullptr, *X0 = nullptr, *lat_qa = nullptr,
          *lat_part = nullptr, *kvx = nullptr;
    uint16_t *qb = nullptr, *xc = nullptr;
    int kvx_cap = 0;
    void *cq = nullptr;
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
    bool adds_again() const { return c.loop_times > 1 && c.loop_stop > c.loop_start; }  // a later pass adds the starting x
};

static WindowShape window_shape(const Layered *l, const LayerDev &L) {
    WindowShape w{};
    w.H = L.d.n_heads, w.G = L.d.n_kv_heads, w.D = L.d.dim, w.V = L.d.vdim;
    w.window = L.d.window, w.rot = L.d.rot_dims, w.gated = L.d.head_gate, w.qk_norm = L.d.qk_norm;
    w.rot_half = L.d.rot_half;
    w.scale = L.d.scale, w.eps = l->c.norm_eps;
    w.seq_len = l->c.seq_len;
    return w;
}
static LatentShape latent_shape(const Layered *l, const LayerDev &L) {
    LatentShape w{};
    w.H = L.d.n_heads, w.D = L.d.dim, w.R = L.d.rot_size, w.V = L.d.vdim, w.C = L.d.kv_rank, w.Q = L.d.q_rank;
    w.rot = L.d.rot_dims, w.rot_half = L.d.rot_half, w.gated = L.d.out_gate;
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
    if (L.d.mixer == L2H_MIX_LATENT) return latent_shape(l, L).n_in();
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
// the same for the keys and values that a latent attention layer's heads make for themselves; all keys are seen
static int latent_tile_size(const Layered *l, const l2h_layer &d) {
    if (l->c.precision) return 0;
    for (int hs : {32, 64, 96, 128, 192})
        if (d.dim + d.rot_size <= hs && d.vdim <= std::min(hs, 128)) return hs;
    return 0;
}
static int latent_tiles(const Layered *l) { return (l->c.seq_len + 31) / 32; }

static int mat_alloc(l2h_model *m, LMat *t, int64_t rows, int K) {
    t->rows = rows;
    t->K = K;
    t->ld = pad64(K);
    return dalloc(m, &t->w, rows * t->ld, true);
}
static LMat mat_rows(const LMat &t, int64_t row0, int64_t rows) {
    LMat v = t;
    v.w = t.w ? t.w + row0 * t.ld : nullptr;
    v.rows = rows;
    return v;
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
        if (d.mixer != L2H_MIX_ATTENTION && d.mixer != L2H_MIX_CHANNEL_DELTA && d.mixer != L2H_MIX_LATENT) return set_err(ctx, L2H_EINVAL, "layer %d: unknown mixer %d", i, d.mixer);
        if (d.n_heads < 1 || d.n_kv_heads < 1 || d.n_heads % d.n_kv_heads != 0)
            return set_err(ctx, L2H_EINVAL, "layer %d: %d heads over %d key/value heads", i, d.n_heads, d.n_kv_heads);
        const int max_head = d.mixer == L2H_MIX_LATENT ? 1024 : 256;
        if (d.dim < 1 || d.dim > max_head || d.vdim < 1 || d.vdim > max_head)
            return set_err(ctx, L2H_EINVAL, "layer %d: head sizes %d, %d (1 to %d are built)", i, d.dim, d.vdim, max_head);
        if ((int64_t)d.n_heads * d.vdim > 32768) return set_err(ctx, L2H_EINVAL, "layer %d: heads x value size above 32768", i);
        if (d.mixer == L2H_MIX_ATTENTION) {
            if (d.window < 1 || std::min(d.window, c.seq_len) > 900000) return set_err(ctx, L2H_EINVAL, "layer %d: window %d", i, d.window);
        } else if (d.mixer == L2H_MIX_LATENT) {
            if (d.n_kv_heads != d.n_heads) return set_err(ctx, L2H_EINVAL, "layer %d: latent attention has a key/value head for every head", i);
            if (d.q_rank < 1 || d.q_rank > 32768 || d.kv_rank < 1 || d.kv_rank > L_LATENT_MAX_RANK || d.rot_size < 0 || d.rot_size > 256)
                return set_err(ctx, L2H_EINVAL, "layer %d: ranks %d, %d, rotated part %d", i, d.q_rank, d.kv_rank, d.rot_size);
            if ((int64_t)d.n_heads * (d.dim + d.rot_size) > 65536) return set_err(ctx, L2H_EINVAL, "layer %d: heads x key size above 65536", i);
        } else if (d.taps < 1 || d.taps > 64 || d.decay_rank < 1 || d.decay_rank > 4096 || d.gate_rank < 1 || d.gate_rank > 4096) {
            return set_err(ctx, L2H_EINVAL, "layer %d: taps %d, ranks %d, %d", i, d.taps, d.decay_rank, d.gate_rank);
        }
        if (d.mixer != L2H_MIX_CHANNEL_DELTA) {
            const int turns = d.mixer == L2H_MIX_LATENT ? d.rot_size : d.dim;
            if (d.rot_dims < 0 || d.rot_dims > turns || d.rot_dims % 2) return set_err(ctx, L2H_EINVAL, "layer %d: %d rotated of %d dimensions", i, d.rot_dims, turns);
            if (d.rot_dims && !(d.rot_base > 0.0)) return set_err(ctx, L2H_EINVAL, "layer %d: rotation base must be positive", i);
            if (d.rot_original > 0.0 && (!(d.rot_factor > 0.0) || !(d.rot_low > 0.0) || !(d.rot_high > d.rot_low)))
                return set_err(ctx, L2H_EINVAL, "layer %d: frequency scaling needs factor > 0 and 0 < low < high", i);
        }
        if (d.ff != L2H_FF_NONE && d.ff != L2H_FF_DENSE && d.ff != L2H_FF_EXPERTS) return set_err(ctx, L2H_EINVAL, "layer %d: unknown feed-forward %d", i, d.ff);
        if (d.ff != L2H_FF_NONE && (d.ff_dim < 1 || d.ff_act < 0 || d.ff_act > L2H_ACT_SILU)) return set_err(ctx, L2H_EINVAL, "layer %d: feed-forward of %d, activation %d", i, d.ff_dim, d.ff_act);
        if (d.ff == L2H_FF_DENSE && d.ff_dim > 36864) return set_err(ctx, L2H_EINVAL, "layer %d: feed-forward of %d is larger than 36864", i, d.ff_dim);
        if (d.ff == L2H_FF_EXPERTS && (d.n_experts < 1 || d.n_experts > 1024 || d.top < 1 || d.top > d.n_experts || d.top > 64 ||
                                       (int64_t)d.top * pad64(d.ff_dim) > 36864))
            return set_err(ctx, L2H_EINVAL, "layer %d: %d of %d experts of %d", i, d.top, d.n_experts, d.ff_dim);
        if (d.ff == L2H_FF_EXPERTS && d.route != L2H_ROUTE_SIGMOID_IN && d.route != L2H_ROUTE_SOFTMAX_OUT)
            return set_err(ctx, L2H_EINVAL, "layer %d: unknown kind of router %d", i, d.route);
    }
    if (c.loop_times < 0 || (c.loop_times > 0 && (c.loop_start < 0 || c.loop_stop <= c.loop_start || c.loop_stop > c.n_layers)))
        return set_err(ctx, L2H_EINVAL, "layers %d to %d run %d times", c.loop_start, c.loop_stop, c.loop_times);
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
    for (int i = 0; i < c.n_layers; i++) {
        const bool again = c.loop_times > 0 && i == c.loop_start;
        for (int t = 0; t < (again ? c.loop_times : 1); t++)
            for (int j = i; j < (again ? c.loop_stop : i + 1); j++) {
                LayerRun r;
                r.layer = j;
                if (again && j == i) r.pass = t;
                l->run.push_back(r);
            }
        if (again) i = c.loop_stop - 1;
    }
    int rc = L2H_OK;
#define A(call) \
    if (rc == L2H_OK) rc = (call)
    A(mat_alloc(m, &l->head, c.vocab_size, c.width));
    A(dalloc(m, &l->final_norm, c.width, true));
    if (c.loop_times) A(dalloc(m, &l->loop_step, (int64_t)c.loop_times * c.width, true));
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
        L.n_plain = mixer_rows(l, L);
        const bool routed = d.parallel && d.ff == L2H_FF_EXPERTS;
        if (routed || L.stacked()) L.n_plain = pad4(L.n_plain);
        L.off_z = L.n_plain;
        if (routed) L.n_plain = pad4(L.off_z + d.n_experts);
        A(mat_alloc(m, &L.in, L.n_plain + (L.stacked() ? L.up_rows() : 0), c.width));
        L.o_cols = pad64(HV);
        L.joined = d.parallel && d.ff == L2H_FF_DENSE && d.mixer == L2H_MIX_LATENT && L.o_cols + d.ff_dim <= 36864;
        A(mat_alloc(m, &L.o, c.width, L.joined ? L.o_cols + d.ff_dim : HV));
        A(dalloc(m, &L.norm1, c.width, true));
        if (d.mixer == L2H_MIX_LATENT) {
            A(mat_alloc(m, &L.uq, d.n_heads * (d.dim + d.rot_size), d.q_rank));
            A(mat_alloc(m, &L.ukv, d.n_heads * (d.dim + d.vdim), d.kv_rank));
            A(dalloc(m, &L.qnorm, d.q_rank, true));
            A(dalloc(m, &L.kvnorm, d.kv_rank, true));
        }
        if (d.mixer != L2H_MIX_CHANNEL_DELTA) {
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
            if (!d.parallel) A(dalloc(m, &L.norm2, c.width, true));
            if (L.stacked())
                L.up = mat_rows(L.in, L.n_plain, L.up_rows());
            else
                A(mat_alloc(m, &L.up, n * L.up_rows(), c.width));
            if (!L.joined) A(mat_alloc(m, &L.down, n * c.width, d.ff_dim));
            if (d.ff == L2H_FF_EXPERTS) {
                if (routed)
                    L.router = mat_rows(L.in, L.off_z, n);
                else
                    A(mat_alloc(m, &L.router, n, c.width));
                if (d.router_bias) A(dalloc(m, &L.router_bias, n, true));
                L.have_gate.assign((size_t)n, 0);
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
    static const char *n[] = {"token embedding", "final norm", "output", "norm 1", "norm 2", "q", "k", "v", "mixer output", "up", "down", "w3",
                              "head gate", "beta", "decay rate", "decay bias", "decay factor in", "decay factor out", "gate factor in",
                              "gate factor out", "mixer norm", "q convolution", "k convolution", "v convolution", "router", "expert up",
                              "expert down", "side embedding", "side gate", "side projection", "side norm", "q down", "q norm", "q up",
                              "k/v down", "k/v norm", "k up", "v up", "output gate", "router bias", "expert gate", "loop step"};
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
    int64_t row0 = 0, row_step = 1, col0 = 0;
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
    case L2H_LOOP_STEP:
        if (!c.loop_times) break;
        vec(l->loop_step, c.width, c.loop_times);
        return L2H_OK;
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
    const bool att = d.mixer == L2H_MIX_ATTENTION, lat = d.mixer == L2H_MIX_LATENT;
    const LatentShape ls = latent_shape(l, L);
    // rows of a feed-forward's input matrix: with a gate, gate and up in turn
    auto pair = [&](int64_t row0, int which) {
        mat(&L.up, d.ff_gated ? 2 * row0 + which : row0, d.ff_dim);
        t.row_step = d.ff_gated ? 2 : 1;
    };
    const DeltaShape ds = delta_shape(l, L);
    const WindowShape ws = window_shape(l, L);
    switch (role) {
    case L2H_RMS_ATT: vec(L.norm1, c.width); return L2H_OK;
    case L2H_RMS_FFN:
        if (!L.norm2) break;
        vec(L.norm2, c.width);
        return L2H_OK;
    case L2H_WQ:
        if (lat) break;
        mat(&L.in, 0, att ? H * D : G * D);
        return L2H_OK;
    case L2H_WK:
        if (lat) break;
        mat(&L.in, att ? ws.off_k() : G * D, G * D);
        return L2H_OK;
    case L2H_WV:
        if (lat) break;
        mat(&L.in, att ? ws.off_v() : 2 * G * D, att ? G * V : H * V);
        return L2H_OK;
    case L2H_WO:
        mat(&L.o, 0, c.width);
        t.e0 = H * V;
        return L2H_OK;
    case L2H_HEAD_GATE:
        if (!att || !d.head_gate) break;
        mat(&L.in, ws.off_g(), H);
        return L2H_OK;
    case L2H_W1:
    case L2H_W3:
        if (d.ff != L2H_FF_DENSE || (role == L2H_W3 && !d.ff_gated)) break;
        pair(0, role == L2H_W3);
        return L2H_OK;
    case L2H_W2:
        if (d.ff != L2H_FF_DENSE) break;
        mat(L.joined ? &L.o : &L.down, 0, c.width);
        t.e0 = d.ff_dim;
        if (L.joined) t.col0 = L.o_cols;
        return L2H_OK;
    case L2H_ROUTER:
        if (d.ff != L2H_FF_EXPERTS) break;
        mat(&L.router, 0, d.n_experts);
        return L2H_OK;
    case L2H_ROUTER_BIAS:
        if (!L.router_bias) break;
        vec(L.router_bias, d.n_experts);
        return L2H_OK;
    case L2H_EXPERT_UP:
    case L2H_EXPERT_GATE:
    case L2H_EXPERT_DOWN:
        if (d.ff != L2H_FF_EXPERTS || (role == L2H_EXPERT_GATE && !d.ff_gated)) break;
        if (expert < 0 || expert >= d.n_experts) return set_err(m->ctx, L2H_EINVAL, "expert %d out of range", expert);
        if (role != L2H_EXPERT_DOWN)
            pair((int64_t)expert * d.ff_dim, role == L2H_EXPERT_UP);
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
    if (lat) switch (role) {
        case L2H_Q_DOWN: mat(&L.in, 0, d.q_rank); return L2H_OK;
        case L2H_Q_NORM: vec(L.qnorm, d.q_rank); return L2H_OK;
        case L2H_Q_UP: mat(&L.uq, 0, H * (D + d.rot_size)); return L2H_OK;
        case L2H_KV_DOWN: mat(&L.in, ls.off_kv(), d.kv_rank + d.rot_size); return L2H_OK;
        case L2H_KV_NORM: vec(L.kvnorm, d.kv_rank); return L2H_OK;
        case L2H_K_UP: mat(&L.ukv, 0, H * D); return L2H_OK;
        case L2H_V_UP: mat(&L.ukv, H * D, H * V); return L2H_OK;
        case L2H_OUT_GATE:
            if (!d.out_gate) break;
            mat(&L.in, ls.off_g(), H * V);
            return L2H_OK;
        }
    if (d.mixer == L2H_MIX_CHANNEL_DELTA) switch (role) {
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
        HIPCHK(ctx, hipMemcpy2D(s.mat->w + s.row0 * s.mat->ld + s.col0, (size_t)(s.mat->ld * s.row_step) * 2, host, (size_t)ne0 * 2,
                                (size_t)ne0 * 2, (size_t)ne1, hipMemcpyHostToDevice));
    }
    if (role == L2H_TOK_EMB || role == L2H_OUTPUT || role == L2H_RMS_FINAL || role == L2H_SIDE_EMB || role == L2H_LOOP_STEP) {
        l->have |= (uint64_t)1 << role;
    } else {
        LayerDev &L = l->layer[(size_t)layer];
        L.have |= (uint64_t)1 << role;
        if (role == L2H_EXPERT_UP) L.have_up[(size_t)expert] = 1;
        if (role == L2H_EXPERT_GATE) L.have_gate[(size_t)expert] = 1;
        if (role == L2H_EXPERT_DOWN) L.have_down[(size_t)expert] = 1;
    }
    return L2H_OK;
}

// ------------------------------------------------------------------------------------------
// state
// ------------------------------------------------------------------------------------------
// floats of what a run of the layer keeps for a sequence: run_state 0 .. 3
static void run_floats(const Layered *l, const LayerDev &L, int64_t n[4]) {
    n[0] = n[1] = n[2] = n[3] = 0;
    if (L.d.mixer == L2H_MIX_ATTENTION) {
        const WindowShape w = window_shape(l, L);
        n[0] = (int64_t)w.G * w.Dp() * w.seq_len;
        n[1] = (int64_t)w.G * w.V * w.seq_len;
    } else if (L.d.mixer == L2H_MIX_LATENT) {
        const LatentShape w = latent_shape(l, L);
        n[0] = (int64_t)w.ld() * w.seq_len;
    } else {
        const DeltaShape s = delta_shape(l, L);
        n[2] = (int64_t)s.taps * s.channels();
        n[3] = (int64_t)s.H * s.D * s.V;
    }
}
static float **run_state(LayerRun &r, int k) {
    float **p[4] = {&r.kc, &r.vc, &r.ring, &r.state};
    return p[k];
}

int layered_finalize(l2h_model *m) {
    l2h_ctx *ctx = m->ctx;
    Layered *l = m->lay;
    const l2h_layered_config &c = l->c;
    int n_in = 1, hv = 1, hid = 1, ne = 1, ssq = 1;
    int64_t part = 1, lq = 0, qa = 0;
    auto missing = [&](uint64_t have, int role, int layer) -> int {
        if (have >> role & 1) return L2H_OK;
        return set_err(ctx, L2H_ESTATE, "missing tensor \"%s\"%s%s", layered_role_name(role), layer >= 0 ? " of layer " : "",
                       layer >= 0 ? std::to_string(layer).c_str() : "");
    };
    int rc;
    for (int r : {L2H_TOK_EMB, L2H_OUTPUT, L2H_RMS_FINAL})
        if ((rc = missing(l->have, r, -1))) return rc;
    if (c.side_dim && (rc = missing(l->have, L2H_SIDE_EMB, -1))) return rc;
    if (c.loop_times && (rc = missing(l->have, L2H_LOOP_STEP, -1))) return rc;
#define DA(p, n, z)                       \
    if ((rc = dalloc(m, &(p), (n), (z)))) \
        return rc;
    for (int i = 0; i < c.n_layers; i++) {
        LayerDev &L = l->layer[(size_t)i];
        const l2h_layer &d = L.d;
        std::vector<int> need = {L2H_RMS_ATT, L2H_WO};
        if (d.mixer == L2H_MIX_LATENT) {
            for (int r : {L2H_Q_DOWN, L2H_Q_NORM, L2H_Q_UP, L2H_KV_DOWN, L2H_KV_NORM, L2H_K_UP, L2H_V_UP}) need.push_back(r);
            if (d.out_gate) need.push_back(L2H_OUT_GATE);
        } else {
            for (int r : {L2H_WQ, L2H_WK, L2H_WV}) need.push_back(r);
        }
        if (d.mixer == L2H_MIX_ATTENTION && d.head_gate) need.push_back(L2H_HEAD_GATE);
        if (d.mixer == L2H_MIX_CHANNEL_DELTA) {
            for (int r : {L2H_BETA, L2H_DECAY_RATE, L2H_DECAY_BIAS, L2H_DECAY_IN, L2H_DECAY_OUT, L2H_GATE_IN, L2H_GATE_OUT, L2H_MIX_NORM,
                          L2H_CONV_Q, L2H_CONV_K, L2H_CONV_V})
                need.push_back(r);
        }
        if (L.norm2) need.push_back(L2H_RMS_FFN);
        if (d.ff == L2H_FF_DENSE) need.push_back(L2H_W1), need.push_back(L2H_W2);
        if (d.ff == L2H_FF_DENSE && d.ff_gated) need.push_back(L2H_W3);
        if (d.ff == L2H_FF_EXPERTS) {
            need.push_back(L2H_ROUTER);
            if (d.router_bias) need.push_back(L2H_ROUTER_BIAS);
            for (int e = 0; e < d.n_experts; e++)
                if (!L.have_up[(size_t)e] || !L.have_down[(size_t)e] || (d.ff_gated && !L.have_gate[(size_t)e])) return set_err(ctx, L2H_ESTATE, "missing expert %d of layer %d", e, i);
        }
        if (c.side_dim)
            for (int r : {L2H_SIDE_GATE, L2H_SIDE_PROJ, L2H_SIDE_NORM}) need.push_back(r);
        for (int r : need)
            if ((rc = missing(L.have, r, i))) return rc;
        if (d.mixer == L2H_MIX_ATTENTION) part = std::max(part, window_part_floats(window_shape(l, L)));
        if (d.mixer == L2H_MIX_LATENT) {
            const LatentShape w = latent_shape(l, L);
            part = std::max(part, latent_part_floats(w, w.H));
            lq = std::max(lq, (int64_t)w.H * w.hq());
            qa = std::max(qa, (int64_t)w.H * w.ld());
        }
        if (d.mixer == L2H_MIX_CHANNEL_DELTA) ssq = std::max(ssq, d.n_heads * delta_splits(d.vdim));
        n_in = std::max(n_in, L.n_plain);
        hv = std::max(hv, std::max(d.n_heads * d.vdim, L.joined ? L.o.ld : 0));
        if (d.ff != L2H_FF_NONE) hid = std::max(hid, d.ff_dim * (d.ff == L2H_FF_EXPERTS ? d.top : 1));
        if (d.ff == L2H_FF_EXPERTS) ne = std::max(ne, d.n_experts);
    }
    for (LayerRun &r : l->run) {
        const LayerDev &L = l->layer[(size_t)r.layer];
        int64_t n[4];
        run_floats(l, L, n);
        for (int k = 0; k < 4; k++)
            if (n[k]) DA(*run_state(r, k), n[k], true);
    }
    if (l->adds_again()) DA(l->x0, c.width, true);
    if (lq) {
        DA(l->lq, lq, true);
        DA(l->qa, qa, true);
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
    for (LayerRun &r : l->run) {
        int64_t n[4];
        run_floats(l, l->layer[(size_t)r.layer], n);
        for (int k = 0; k < 4; k++)
            if (n[k]) HIPCHK(m->ctx, hipMemsetAsync(*run_state(r, k), 0, (size_t)n[k] * 4, s));
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

// The residual stream moves to the other of its two buffers where a layer's pending per-token update is applied by the launch
// that reads it next; it ends in m->x.  (Before a pass of a loop the update is applied where the stream lies.)
struct Stream {
    l2h_model *m;
    float *x;
    const float *yw = nullptr;  // the update l->y is pending, with these weights
    explicit Stream(l2h_model *model) : m(model) {
        const Layered *l = m->lay;
        int moves = 0;
        for (size_t r = 0; l->c.side_dim && r < l->run.size(); r++)
            if (r + 1 == l->run.size() || l->run[r + 1].pass < 0) moves++;
        x = moves & 1 ? l->x_alt : m->x;
    }
    // norm of the stream and a matrix
    RowsArgs normed(const LMat &w, const float *normw, float *out) {
        const Layered *l = m->lay;
        RowsArgs a = rows_of(w, x, out);
        a.normw = normw;
        a.eps = l->c.norm_eps;
        if (yw) {
            a.y = l->y;
            a.yw = yw;
            a.mult = l->c.residual_mult;
            a.x_out = x = x == m->x ? l->x_alt : m->x;
            yw = nullptr;
        }
        return a;
    }
};

hipError_t layered_output(l2h_model *m) {
    Layered *l = m->lay;
    RowsArgs a = rows_of(l->head, m->x, m->logits);
    a.normw = l->final_norm;
    a.eps = l->c.norm_eps;
    return k_rows(m->ctx->stream, a, RP_NORM, RE_STORE, m->ctx->prop.multiProcessorCount);
}

static hipError_t step_latent(l2h_model *m, const LayerDev &L, const LayerRun &run, int cu) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const LatentShape w = latent_shape(l, L);
    hipError_t e;
    RowsArgs q = rows_of(L.uq, l->in, l->lq);
    q.normw = L.qnorm;
    q.eps = w.eps;
    CK(k_rows(s, q, RP_NORM, RE_STORE, cu));
    CK(k_latent_query(s, w, L.freq, l->lq, L.ukv.w, L.ukv.ld, l->qa, 1, 0, m->ctl, l->in, L.kvnorm, run.kc));
    CK(k_latent_attend(s, w, l->qa, run.kc, l->part, 1, 0, m->ctl));
    const int64_t cols = L.joined ? L.o_cols : w.H * w.V;
    return k_latent_value(s, w, l->part, L.ukv.w, L.ukv.ld, l->in, 0, 1, l->mix, cols, cols, 1);
}

hipError_t layered_enqueue_token(l2h_model *m) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const int cu = m->ctx->prop.multiProcessorCount;
    const l2h_layered_config &c = l->c;
    hipError_t e;
    Stream st(m);
    CK(k_embed(s, m->glob[L2H_TOK_EMB], m->ctl, m->prompt_dev, st.x, m->rope_cs, 0, 1.0f, c.embed_scale, l->x0));
    for (const LayerRun &run : l->run) {
        LayerDev &L = l->layer[(size_t)run.layer];
        const l2h_layer &d = L.d;
        if (run.pass >= 0) {
            if (st.yw) CK(k_norm_rows(s, st.x, c.width, 1, nullptr, c.norm_eps, l->y, st.yw, c.residual_mult, nullptr, nullptr, 0, 1));
            st.yw = nullptr;
            CK(k_stream_add(s, st.x, run.pass ? l->x0 : nullptr, l->loop_step + (int64_t)run.pass * c.width, 1, c.width));
        }
        RowsArgs in = st.normed(L.in, L.norm1, l->in);
        float *x = st.x;
        const bool early = d.parallel;  // the feed-forward reads the mixer's input
        if (L.stacked()) {
            in.glu_from = L.n_plain;
            in.act = d.ff_act;
            in.out2 = L.joined ? l->mix + L.o_cols : l->hid;
            CK(k_rows(s, in, RP_NORM, RE_STORE_GLU, cu));
        } else {
            CK(k_rows(s, in, RP_NORM, RE_STORE, cu));
        }
        RowsArgs o = rows_of(L.o, l->mix, x);
        o.resid = x;
        o.mult = c.residual_mult;
        int o_pro = RP_PLAIN;
        if (d.mixer == L2H_MIX_ATTENTION) {
            CK(k_window_step(s, window_shape(l, L), L.freq, l->in, run.kc, run.vc, m->ctl, l->part, l->mix));
        } else if (d.mixer == L2H_MIX_LATENT) {
            CK(step_latent(m, L, run, cu));
        } else {
            const DeltaWeights w = {L.conv, L.rate, L.bias, L.a2.w, L.g2.w, L.a2.ld, L.g2.ld};
            CK(k_delta_step(s, delta_shape(l, L), w, l->in, run.ring, run.state, m->ctl, l->mix, l->ssq, l->gate));
            o.normw = L.mixnorm;
            o.eps = c.norm_eps;
            o.ssq = l->ssq;
            o.gate = l->gate;
            o.hv = d.vdim;
            o.n_split = delta_splits(d.vdim);
            o_pro = RP_HEADNORM;
        }
        if (!early || d.ff == L2H_FF_NONE || (L.stacked() && L.joined)) CK(k_rows(s, o, o_pro, RE_RESID, cu));
        if (d.ff != L2H_FF_NONE && !(L.stacked() && L.joined)) {
            RowsArgs up = rows_of(L.up, x, l->hid), down = rows_of(L.down, l->hid, x);
            up.normw = early ? L.norm1 : L.norm2;
            up.eps = c.norm_eps;
            up.act = d.ff_act;
            down.resid = x;
            down.mult = c.residual_mult;
            if (d.ff == L2H_FF_DENSE) {
                if (L.joined) up.out = l->mix + L.o_cols;
                if (!L.stacked()) CK(k_rows(s, up, RP_NORM, d.ff_gated ? RE_GLU : RE_ACT, cu));
                if (early) CK(k_rows(s, o, o_pro, RE_RESID, cu));
                if (!L.joined) CK(k_rows(s, down, RP_PLAIN, RE_RESID, cu));
            } else {
                RowsArgs r = rows_of(L.router, x, l->z);
                r.normw = up.normw;
                r.eps = c.norm_eps;
                if (!early) CK(k_rows(s, r, RP_NORM, RE_STORE, cu));
                for (RowsArgs *a : {&up, &down}) {
                    a->z = early ? l->in + L.off_z : l->z;
                    a->z_bias = L.router_bias;
                    a->n_experts = d.n_experts;
                    a->top = d.top;
                    a->route = d.route;
                }
                up.rows_each = L.up_rows();
                up.n_rows = (int64_t)d.top * L.up_rows();
                down.rows_each = c.width;
                down.n_rows = c.width;
                CK(k_rows(s, up, RP_UP, d.ff_gated ? RE_GLU : RE_UP, cu));
                if (early) CK(k_rows(s, o, o_pro, RE_RESID, cu));
                CK(k_rows(s, down, RP_DOWN, RE_RESID, cu));
            }
        }
        if (c.side_dim) {
            RowsArgs g = rows_of(L.side_gate, x, l->se);
            g.act = LACT_GELU_TANH;
            g.emb = l->side_emb + (int64_t)run.layer * c.side_dim;
            g.emb_ld = (int64_t)c.n_layers * c.side_dim;
            g.ctl = m->ctl;
            g.prompt = m->prompt_dev;
            CK(k_rows(s, g, RP_PLAIN, RE_EMBED, cu));
            CK(k_rows(s, rows_of(L.side_proj, l->se, l->y), RP_PLAIN, RE_STORE, cu));
            st.yw = L.side_norm;
        }
    }
    CK(k_rows(s, st.normed(l->head, l->final_norm, m->logits), RP_NORM, RE_STORE, cu));
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
        if (L.d.ff == L2H_FF_DENSE) add(&L.up, L.up_rows(), 1);
        if (L.d.ff == L2H_FF_EXPERTS) {
            if (std::min(L.up_rows(), l->W()) < L_IMAGE_MIN_ROWS) continue;  // (both or neither)
            add(&L.up, L.up_rows(), L.d.n_experts);
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
        DA(l->kept, (int64_t)l->run.size() * cap * c.width);
        l->kept_cap = cap;
    }
    if (l->cap >= cap) return L2H_OK;
    int64_t n_in = 1, ch = 1, g = 1, h = 1, hd = 1, hv = 1, lhv = 64, lra = 64, lrg = 64, hid = 64, ne = 1, slots = 1, up_slots = 1, tiles = 1;
    int64_t kvt = 0, rec = 0, qb = 0, xc = 0, kvx = 0, cq = 0, lat_qa = 0, lat_part = 0;
    // tokens of a block of latent attention: few where longer prompts go another way
    const int lat_block = std::min(cap, L_LATENT_BLOCK), kvx_cap = std::min((c.seq_len + 255) / 256 * 256, 2048);
    bool moe = false;
    for (LayerDev &L : l->layer) {
        const l2h_layer &d = L.d;
        n_in = std::max<int64_t>(n_in, L.n_plain);
        hv = std::max<int64_t>(hv, d.n_heads * d.vdim);
        lhv = std::max<int64_t>(lhv, L.o.ld);
        if (d.mixer == L2H_MIX_ATTENTION) {
            ch = std::max<int64_t>(ch, d.n_heads * d.dim);
            const int hs = attention_tile_size(d);
            if (hs && !c.precision) {
                ch = std::max<int64_t>(ch, d.n_heads * hs);
                kvt = std::max<int64_t>(kvt, (int64_t)d.n_kv_heads * attention_tiles(l, L, cap) * k_pf_kv_tile_bytes(hs));
            }
        } else if (d.mixer == L2H_MIX_LATENT) {
            const LatentShape w = latent_shape(l, L);
            const int hs = latent_tile_size(l, d);
            const int64_t block = hs ? std::min(lat_block, L_LATENT_SMALL) : lat_block;
            ch = std::max<int64_t>(ch, w.H * w.hq());
            cq = std::max<int64_t>(cq, L.uq.ld);
            lat_qa = std::max(lat_qa, block * w.H * w.ld());
            for (int64_t k = 1; k <= block; k++) lat_part = std::max(lat_part, latent_part_floats(w, k * w.H));
            if (hs) {
                qb = std::max<int64_t>(qb, w.H * hs);
                xc = std::max<int64_t>(xc, L.ukv.ld);
                kvx = std::max<int64_t>(kvx, L.ukv.rows);
                kvt = std::max<int64_t>(kvt, (int64_t)w.H * latent_tiles(l) * k_pf_kv_tile_bytes(hs));
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
        if (d.ff == L2H_FF_DENSE && !L.joined) hid = std::max<int64_t>(hid, L.down.ld);
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
    if (cq) {
        DB(l->cq, cap * cq);
        DA(l->lat_qa, lat_qa);
        DA(l->lat_part, lat_part);
    }
    if (qb) {
        DA(l->qb, cap * qb);
        DA(l->xc, kvx_cap * xc);
        DA(l->kvx, kvx_cap * kvx);
        l->kvx_cap = kvx_cap;
    }
    if (l->adds_again()) DA(l->X0, (int64_t)cap * c.width);
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
static hipError_t to_acts(l2h_model *m, GemmArgs a, int epi, void *out, int64_t lda, const LMat *w = nullptr, int64_t cols = 0) {
    a.outa = out;
    a.lda = lda;
    a.acols = cols;
    if (w && image_takes(*w, a.M)) {
        a.w = w->image;
        return k_tiles(m->ctx->stream, a, epi);
    }
    return k_gemm(m->ctx->stream, a, m->lay->c.precision, epi);
}

static hipError_t prompt_delta(l2h_model *m, LayerDev &L, const LayerRun &run, int M, int pos0) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const int prec = l->c.precision;
    const DeltaShape d = delta_shape(l, L);
    const int64_t ldr = L.n_plain, hd = d.H * d.D, hv = d.H * d.V;
    hipError_t e;
    CK(k_delta_prepare(s, d, L.conv, l->raw, ldr, run.ring, M, pos0, l->qkv, l->kq, l->beta, l->fa, L.a2.ld, l->fg, L.g2.ld, prec));
    CK(k_delta_ring(s, d, l->raw, ldr, run.ring, M, pos0));
    GemmArgs a = gemm_of(L.a2, l->fa, M);
    a.outf = l->lg;
    a.ldo = hd;
    a.rate = L.rate;
    a.bias = L.bias;
    a.hd = d.D;
    CK(k_gemm(s, a, prec, GE_DECAY));
    CK(product(m, gemm_of(L.g2, l->fg, M), GE_SIGMOID, l->gt, hv, 1.0f));
    if (M >= L_DELTA_WALK_MIN)
        CK(k_delta_walk(s, d, l->qkv, l->beta, l->lg, run.state, M, pos0, l->rec, l->ob));
    else
        CK(k_delta_scan(s, d, l->qkv, l->kq, l->beta, l->lg, run.state, M, pos0, l->ob));
    CK(k_head_norm_rows(s, l->ob, l->gt, L.mixnorm, M, d.H, d.V, d.eps, l->ao, L.o.ld, prec));
    return hipSuccess;
}

static hipError_t prompt_attention(l2h_model *m, LayerDev &L, const LayerRun &run, int M, int pos0) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const WindowShape w = window_shape(l, L);
    const int64_t ldr = L.n_plain;
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
        CK(k_window_prepare(s, w, L.freq, l->raw, ldr, run.kc, run.vc, M, pos0, nullptr, qb, hs));
        CK(k_pf_kv_tiles(s, run.kc, run.vc, l->kvt, n_tiles, cap, hs, w.G, w.seq_len, win.tile0, w.Dp(), w.V));
        return k_pf_attention(s, qb, (uint16_t *)l->ao, l->kvt, cap, M, pos0, hs, w.H, w.G, w.H * hs, &win);
    }
    CK(k_window_prepare(s, w, L.freq, l->raw, ldr, run.kc, run.vc, M, pos0, l->qkv, nullptr, 0));
    CK(k_window_rows(s, w, l->qkv, l->raw, ldr, run.kc, run.vc, M, pos0, l->ao, L.o.ld, l->c.precision));
    return hipSuccess;
}

static hipError_t prompt_latent(l2h_model *m, LayerDev &L, const LayerRun &run, int M, int pos0) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const LatentShape w = latent_shape(l, L);
    const int64_t ldr = L.n_plain, ldq = w.H * w.hq(), ldkv = L.ukv.rows, lda = L.o.ld;
    const int prec = l->c.precision, hs = latent_tile_size(l, L.d);
    hipError_t e;
    CK(k_latent_prepare(s, w, L.qnorm, L.kvnorm, L.freq, l->raw, ldr, run.kc, M, pos0, l->cq, L.uq.ld, prec));
    CK(product(m, gemm_of(L.uq, l->cq, M), GE_STORE, l->qkv, ldq, 1.0f));
    if (!hs || M <= L_LATENT_SMALL) {
        const int block = std::min(std::min(l->cap, L_LATENT_BLOCK), hs ? L_LATENT_SMALL : M);
        for (int m0 = 0; m0 < M; m0 += block) {
            const int n = std::min(block, M - m0);
            void *out = (char *)l->ao + (int64_t)m0 * lda * l->asize();
            CK(k_latent_query(s, w, L.freq, l->qkv + m0 * ldq, L.ukv.w, L.ukv.ld, l->lat_qa, n, pos0 + m0, nullptr, nullptr, nullptr, nullptr));
            CK(k_latent_attend(s, w, l->lat_qa, run.kc, l->lat_part, n, pos0 + m0, nullptr));
            CK(k_latent_value(s, w, l->lat_part, L.ukv.w, L.ukv.ld, l->raw + m0 * ldr, ldr, n, out, lda, L.o_cols, prec));
        }
        return hipSuccess;
    }
    CK(k_latent_heads(s, w, L.freq, l->qkv, l->qb, hs, M, pos0));
    const int tiles = latent_tiles(l);
    for (int p = 0; p < pos0 + M; p += l->kvx_cap) {  // the heads' own keys and values, from the cached latents
        const int n = std::min(l->kvx_cap, pos0 + M - p);
        CK(k_latent_rows(s, w, run.kc, p, n, l->xc, L.ukv.ld));
        CK(product(m, gemm_of(L.ukv, l->xc, n), GE_STORE, l->kvx, ldkv, 1.0f));
        CK(k_pf_row_tiles(s, l->kvx, ldkv, run.kc + w.Cp(), w.ld(), w.R, l->kvt, p, n, tiles, hs, w.H, w.D, w.V));
    }
    PfWindow win;
    win.window = l->c.seq_len;  // (every key)
    win.vdim = w.V;
    win.scale = w.scale;
    win.gate = w.gated ? l->raw + w.off_g() : nullptr;
    win.gate_each = 1;
    win.ldg = ldr;
    win.ldo = lda;
    win.cols = L.o_cols;
    return k_pf_attention(s, l->qb, (uint16_t *)l->ao, l->kvt, tiles, M, pos0, hs, w.H, w.H, w.H * hs, &win);
}

static hipError_t prompt_experts(l2h_model *m, LayerDev &L, int M) {
    Layered *l = m->lay;
    hipStream_t s = m->ctx->stream;
    const l2h_layer &d = L.d;
    const int prec = l->c.precision;
    hipError_t e;
    if (!d.parallel) CK(product(m, gemm_of(L.router, l->xn, M), GE_STORE, l->zb, d.n_experts, 1.0f));
    // (a parallel layer's logits are among the products of the mixer's input)
    CK(k_route(s, d.parallel ? l->raw + L.off_z : l->zb, d.parallel ? L.n_plain : d.n_experts, L.router_bias, M, d.n_experts, d.top, d.route,
               l->choice, l->score));
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
    const int epi = d.ff_gated ? GE_GLU : GE_UP;
    up.n_rows = L.up_rows();
    up.expert_stride = (int64_t)L.up_rows() * L.up.ld;
    up.gather = l->slot_row;
    up.row_scale = l->slot_scale;
    up.scale_in = d.route == L2H_ROUTE_SIGMOID_IN;
    up.act = d.ff_act;
    up.outa = l->hb;
    up.lda = L.down.ld;
    if (image) {
        up.w = L.up.image;
        up.expert_stride = L.up.image_stride;
        CK(k_tiles(s, up, epi));
    } else {
        CK(k_gemm(s, up, prec, epi));
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
    CK(k_pf_embed(s, m->glob[L2H_TOK_EMB], l->tok, l->X, M, c.embed_scale, l->X0));
    const float *py = nullptr, *pyw = nullptr;  // per-token update that waits for the next reader of the residual stream
    auto keep = [&](int r) -> hipError_t {
        if (!l->keep || r < 0) return hipSuccess;
        return hipMemcpyAsync(l->kept + ((int64_t)r * l->kept_cap) * W, l->X, (size_t)M * W * 4, hipMemcpyDeviceToDevice, s);
    };
    for (int r = 0; r < (int)l->run.size(); r++) {
        const LayerRun &run = l->run[(size_t)r];
        LayerDev &L = l->layer[(size_t)run.layer];
        const l2h_layer &d = L.d;
        bool kept = false;
        if (run.pass >= 0) {
            if (py) CK(k_norm_rows(s, l->X, W, M, nullptr, eps, py, pyw, mult, nullptr, nullptr, 0, prec));
            py = nullptr;
            CK(keep(r - 1));
            kept = true;
            CK(k_stream_add(s, l->X, run.pass ? l->X0 : nullptr, l->loop_step + (int64_t)run.pass * W, M, W));
        }
        CK(k_norm_rows(s, l->X, W, M, L.norm1, eps, py, pyw, mult, nullptr, l->xn, ldw, prec));
        py = nullptr;
        if (!kept) CK(keep(r - 1));
        CK(product(m, gemm_of(mat_rows(L.in, 0, L.n_plain), l->xn, M), GE_STORE, l->raw, L.n_plain, 1.0f));
        CK(d.mixer == L2H_MIX_ATTENTION ? prompt_attention(m, L, run, M, pos0)
           : d.mixer == L2H_MIX_LATENT  ? prompt_latent(m, L, run, M, pos0)
                                        : prompt_delta(m, L, run, M, pos0));
        GemmArgs up = gemm_of(L.up, l->xn, M);
        up.act = d.ff_act;
        const int up_epi = d.ff_gated ? GE_GLU : GE_ACT;
        if (L.joined) CK(to_acts(m, up, up_epi, (char *)l->ao + (int64_t)L.o_cols * l->asize(), L.o.ld, &L.up, L.o.ld - L.o_cols));
        CK(product(m, gemm_of(L.o, l->ao, M), GE_RESID, l->X, W, mult));
        if (d.ff != L2H_FF_NONE && !L.joined) {
            if (!d.parallel) CK(k_norm_rows(s, l->X, W, M, L.norm2, eps, nullptr, nullptr, mult, nullptr, l->xn, ldw, prec));
            if (d.ff == L2H_FF_DENSE) {
                CK(to_acts(m, up, up_epi, l->hb, L.down.ld, &L.up));
                CK(product(m, gemm_of(L.down, l->hb, M), GE_RESID, l->X, W, mult));
            } else {
                CK(prompt_experts(m, L, M));
            }
        }
        if (c.side_dim) {
            CK(k_norm_rows(s, l->X, W, M, nullptr, eps, nullptr, nullptr, mult, nullptr, l->xn, ldw, prec));
            GemmArgs g = gemm_of(L.side_gate, l->xn, M);
            g.act = LACT_GELU_TANH;
            g.emb = l->side_emb + (int64_t)run.layer * c.side_dim;
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
    CK(keep((int)l->run.size() - 1));
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
    if (!l->kept || layer < 0 || layer >= (int)l->run.size() || n != (int64_t)l->kept_n * l->c.width)
        return set_err(m->ctx, L2H_EINVAL, "kept residual stream: layer %d, %lld floats (holds %d positions)", layer, (long long)n, l->kept_n);
    HIPCHK(m->ctx, hipStreamSynchronize(m->ctx->stream));
    HIPCHK(m->ctx, hipMemcpy(host, l->kept + (int64_t)layer * l->kept_cap * l->c.width, (size_t)n * 4, hipMemcpyDeviceToHost));
    return L2H_OK;
}
