// engine_decoder.hip -- the layered-decoder family of libpgmi: a text model described as a list of layers, each a
// mixer and an optional feed-forward, around residual streams or one plain residual.  Weight layout, derived
// tensors, the per-sequence state slab, the ragged forward (prompts and portions of prompts) and the decode step
// (hipGraph-replayed), over the mechanisms of decoder.h.  A design is its layer list and constants; nothing here names one.
#include <set>

#include "decoder.h"
#include "engine.h"

namespace {

int r8(int n) { return (n + 7) & ~7; }

// a projection as the kernels read it: [n][ldw] rows, k columns (a multiple of 8, zero past the true width)
struct Lin {
    const uint16_t* w = nullptr;
    int n = 0, k = 0, ldw = 0;
};

struct Sub {  // one residual sublayer's stream weights (null: plain residual) and norm
    const uint16_t *in, *out, *mix, *norm;
};

struct LayerW {
    Sub sub[2];
    Lin in;    // mamba1: in; attention: q|k|v; mingru: z|x|g
    Lin x, dt;  // mamba1
    Lin o;
    Lin gu, down;  // feed-forward, or the shared expert
    Lin router;    // with the shared expert's gate as its last row
    Lin egu, ed;   // every expert's gate|up and down, expert after expert
    const uint16_t *correction = nullptr, *canon = nullptr;
    const double* turns = nullptr;  // rotary: turns per position of every pair
    const uint16_t* bias = nullptr;  // of `in`
    const uint16_t *conv = nullptr, *conv_b = nullptr, *dt_b = nullptr, *A_log = nullptr, *D = nullptr, *r1 = nullptr,
                   *r2 = nullptr;
};

struct StateAt {  // byte offsets of a layer's regions in the state slab
    int64_t a = 0, b = 0;  // mamba1: taps, scan state; attention: keys, values; mingru: state
    int64_t ring = 0;      // last inputs of the input convolution
};
struct StateMap {
    std::vector<StateAt> at;
    int64_t history = 0;  // tokens by position, where the embedding reads pairs
    int64_t bytes = 0;
};

}  // namespace

struct DecoderState {
    pgmi_decoder_config c;
    std::vector<pgmi_layer_spec> L;
    std::vector<LayerW> W;
    Act act;
    int es;  // bytes per activation element
    const uint16_t *embed = nullptr, *fnorm = nullptr, *pairs = nullptr;
    Lin head;
    std::vector<void*> derived;  // padded weights, joined biases
    // workspace of `rows` rows, `chunks` scan chunks and `gchunks` chunks of the gated recurrence
    int rows = 0, chunks = 0, gchunks = 0;
    void* arena = nullptr;
    float *X = nullptr, *slabs = nullptr, *dt = nullptr, *bc = nullptr, *cstate = nullptr, *csum = nullptr;
    uint8_t *h = nullptr, *p0 = nullptr, *p1 = nullptr, *p2 = nullptr, *dtl = nullptr;
    // mixture of experts: activations and outputs per entry, choices, weights, gates, lists, counters, used experts
    uint8_t *ea = nullptr, *ey = nullptr;
    float *inv = nullptr, *ew = nullptr, *egate = nullptr;
    int *esel = nullptr, *elist = nullptr, *ecnt = nullptr, *eactive = nullptr;
    int zero_words = 0;  // the counters and the number of used experts
    size_t slab_bytes = 0;
    int ldh = 0, ld0 = 0, ld1 = 0, ld2 = 0, ldd = 0;
    // step metadata
    void* meta = nullptr;
    size_t meta_bytes = 0;
    std::vector<int> host;
    // decode
    int *slot = nullptr, *pos = nullptr;  // [max_batch]
    float* part = nullptr;                // attention partials
    size_t part_floats = 0;
    float* pmax = nullptr;
    int* pidx = nullptr;
    int64_t *d_ids = nullptr, *d_next = nullptr;
    std::vector<int> known_slot, known_pos;  // what slot / pos hold once the enqueued steps have run (empty: unknown)
};

namespace {

std::string lname(int i, const char* s) { return "l" + std::to_string(i) + "." + s; }

// add_slot without the 256-byte rounding, for the tensors whose rows one projection joins
void add_joined(pgmi_ctx* x, const std::vector<std::pair<std::string, std::vector<int64_t>>>& ts) {
    for (const auto& t : ts) {
        Slot s;
        s.name = t.first;
        s.ndim = (int)t.second.size();
        s.numel = 1;
        for (int i = 0; i < 4; ++i) {
            s.shape[i] = i < s.ndim ? t.second[i] : 1;
            s.numel *= s.shape[i];
        }
        s.off = x->slab_bytes;
        x->slab_bytes += s.numel * 2;
        x->index[s.name] = (int)x->slots.size();
        x->slots.push_back(s);
    }
    x->slab_bytes = (x->slab_bytes + 255) / 256 * 256;
}

int qkv_rows(const pgmi_layer_spec& l) { return l.heads * l.dim + (l.kv_from < 0 ? l.kv_heads * (l.dim + l.vdim) : 0); }
bool has_ff(const pgmi_layer_spec& l) { return l.ff > 0 || l.experts > 0; }

void build_decoder_layout(pgmi_ctx* x) {
    const DecoderState& d = *x->dec;
    const int64_t D = d.c.width, S = d.c.streams;
    auto add_norm = [&](const std::string& name) {
        if (d.c.norm_scalar) add_slot(x, name, {});
        else add_slot(x, name, {D});
    };
    add_slot(x, "embed", {d.c.vocab, D});
    if (d.c.untied_head) add_slot(x, "head", {d.c.vocab, D});
    if (d.c.bigram_buckets) add_slot(x, "bigram", {(int64_t)d.c.bigram_buckets + 1, D});
    for (int i = 0; i < d.c.n_layers; ++i) {
        const pgmi_layer_spec& l = d.L[i];
        for (int q = 1; q <= (has_ff(l) ? 2 : 1); ++q) {
            const std::string n = std::to_string(q);
            add_norm(lname(i, "norm") + n);
            if (d.c.plain_residual) continue;
            add_slot(x, lname(i, "hc") + n + ".in", {S});
            add_slot(x, lname(i, "hc") + n + ".out", {S});
            add_slot(x, lname(i, "hc") + n + ".mix", {S, S});
        }
        if (d.c.canon_taps) add_slot(x, lname(i, "canon1"), {D, d.c.canon_taps});
        if (l.mixer == PGMI_MIXER_MAMBA1) {
            const int64_t C = l.inner, N = l.state, R = l.dt_rank;
            add_slot(x, lname(i, "mix.in"), {2 * C, D});
            add_slot(x, lname(i, "mix.conv"), {C, l.conv});
            add_slot(x, lname(i, "mix.conv.b"), {C});
            add_slot(x, lname(i, "mix.x"), {R + 2 * N, C});
            add_slot(x, lname(i, "mix.dt"), {C, R});
            add_slot(x, lname(i, "mix.dt.b"), {C});
            add_slot(x, lname(i, "mix.A_log"), {C, N});
            add_slot(x, lname(i, "mix.D"), {C});
            add_slot(x, lname(i, "mix.o"), {D, C});
        } else if (l.mixer == PGMI_MIXER_ATTENTION) {
            const int64_t q = (int64_t)l.heads * l.dim, k = (int64_t)l.kv_heads * l.dim, v = (int64_t)l.kv_heads * l.vdim;
            if (l.kv_from < 0) {
                add_joined(x, {{lname(i, "mix.q"), {q, D}}, {lname(i, "mix.k"), {k, D}}, {lname(i, "mix.v"), {v, D}}});
                if (l.proj_bias)
                    add_joined(x, {{lname(i, "mix.q.b"), {q}}, {lname(i, "mix.k.b"), {k}}, {lname(i, "mix.v.b"), {v}}});
            } else {
                add_slot(x, lname(i, "mix.q"), {q, D});
                if (l.proj_bias) add_slot(x, lname(i, "mix.q.b"), {q});
            }
            if (l.distance_bias) {
                add_slot(x, lname(i, "mix.r1"), {l.heads});
                add_slot(x, lname(i, "mix.r2"), {l.heads});
            }
            add_slot(x, lname(i, "mix.o"), {D, (int64_t)l.heads * l.vdim});
        } else {
            const int64_t C = l.width;
            add_joined(x, {{lname(i, "mix.z"), {C, D}}, {lname(i, "mix.x"), {C, D}}, {lname(i, "mix.g"), {C, D}}});
            add_joined(x, {{lname(i, "mix.z.b"), {C}}, {lname(i, "mix.x.b"), {C}}});
            add_slot(x, lname(i, "mix.o"), {D, C});
        }
        if (l.ff) {
            add_joined(x, {{lname(i, "mlp.gate"), {l.ff, D}}, {lname(i, "mlp.up"), {l.ff, D}}});
            add_slot(x, lname(i, "mlp.down"), {D, l.ff});
        }
        if (l.experts) {
            const int64_t n = l.experts + l.identity;
            std::vector<std::pair<std::string, std::vector<int64_t>>> gu, down, router = {{lname(i, "mlp.router"), {n, D}}};
            for (int e = 0; e < l.experts; ++e) {
                const std::string at = lname(i, "mlp.e") + std::to_string(e);
                gu.push_back({at + ".gate", {l.expert_ff, D}});
                gu.push_back({at + ".up", {l.expert_ff, D}});
                down.push_back({at + ".down", {D, l.expert_ff}});
            }
            add_joined(x, gu);
            add_joined(x, down);
            if (l.shared_ff) router.push_back({lname(i, "mlp.shared.sg"), {1, D}});
            add_joined(x, router);
            add_slot(x, lname(i, "mlp.correction"), {n});
            if (l.shared_ff) {
                add_joined(x, {{lname(i, "mlp.shared.gate"), {l.shared_ff, D}}, {lname(i, "mlp.shared.up"), {l.shared_ff, D}}});
                add_slot(x, lname(i, "mlp.shared.down"), {D, l.shared_ff});
            }
        }
    }
    if (d.c.norm_scalar) add_slot(x, "final.norm", {});
    else add_slot(x, "final.norm", {D});
}

// the state slab's regions for n_slots sequences of up to max_tokens
StateMap state_layout(const DecoderState& d, int n_slots, int max_tokens) {
    StateMap m;
    auto take = [&](int64_t bytes) {
        const int64_t o = m.bytes;
        m.bytes += (bytes + 255) / 256 * 256;
        return o;
    };
    m.at.assign(d.c.n_layers, {});
    for (int i = 0; i < d.c.n_layers; ++i) {
        const pgmi_layer_spec& l = d.L[i];
        StateAt& s = m.at[i];
        if (l.mixer == PGMI_MIXER_MAMBA1) {
            s.a = take((int64_t)n_slots * (l.conv - 1) * l.inner * 4);
            s.b = take((int64_t)n_slots * l.inner * l.state * 4);
        } else if (l.mixer == PGMI_MIXER_ATTENTION && l.kv_from < 0) {
            s.a = take((int64_t)n_slots * l.kv_heads * max_tokens * r8(l.dim) * d.es);
            s.b = take((int64_t)n_slots * l.kv_heads * max_tokens * r8(l.vdim) * d.es);
        } else if (l.mixer == PGMI_MIXER_ATTENTION) {
            s.a = m.at[l.kv_from].a;
            s.b = m.at[l.kv_from].b;
        } else {
            s.a = take((int64_t)n_slots * l.width * 4);
        }
        if (d.c.canon_taps > 1) s.ring = take((int64_t)n_slots * d.c.canon_taps * d.c.width * 4);
    }
    if (d.c.bigram_buckets) m.history = take((int64_t)n_slots * max_tokens * 4);
    return m;
}

int64_t decoder_state_bytes(const pgmi_ctx* x, int batch, int max_tokens) {
    return state_layout(*x->dec, batch, max_tokens).bytes;
}

int derived_alloc(DecoderState& d, uint16_t** p, size_t elems) {
    void* q = nullptr;
    if (hipMalloc(&q, std::max<size_t>(elems, 128) * 2) != hipSuccess)
        return fail(PGMI_E_NOMEM, "derived weights");
    d.derived.push_back(q);
    *p = reinterpret_cast<uint16_t*>(q);
    return 0;
}

// W [n][k] as stored; a padded copy when a row is not a whole number of 16-byte pieces
int make_lin(DecoderState& d, const uint16_t* w, int n, int k, Lin* out) {
    *out = {w, n, r8(k), k};
    if (k % 8 == 0) return 0;
    uint16_t* p;
    int rc;
    if ((rc = derived_alloc(d, &p, (size_t)n * r8(k)))) return rc;
    pad_rows(nullptr, w, n, k, r8(k), p);
    *out = {p, n, r8(k), r8(k)};
    return 0;
}

// turns per position of the rotated pairs: base^(-2i / dims) over a full turn, scaled by wavelength
int make_turns(DecoderState& d, const pgmi_layer_spec& l, const double** out) {
    if (!l.rot_dims) return 0;
    constexpr double kTurn = 6.283185307179586476925286766559;
    std::vector<double> t;
    for (int i = 0; i < l.rot_dims / 2; ++i) {
        double f = std::pow(l.rot_base, -2.0 * i / l.rot_dims);
        if (l.rot_original > 0) {
            const double wave = kTurn / f;
            if (wave > l.rot_original / l.rot_low) {
                f /= l.rot_factor;
            } else if (!(wave < l.rot_original / l.rot_high)) {
                const double s = (l.rot_original / wave - l.rot_low) / (l.rot_high - l.rot_low);
                f = (1.0 - s) * f / l.rot_factor + s * f;
            }
        }
        t.push_back(f / kTurn);
    }
    uint16_t* p;
    int rc;
    if ((rc = derived_alloc(d, &p, t.size() * 4))) return rc;
    HIPCHK(hipMemcpy(p, t.data(), t.size() * sizeof(double), hipMemcpyHostToDevice));
    *out = reinterpret_cast<const double*>(p);
    return 0;
}

void drop_derived(DecoderState& d) {
    for (void* p : d.derived) (void)hipFree(p);
    d.derived.clear();
}

int decoder_prepare(pgmi_ctx* x) {
    DecoderState& d = *x->dec;
    HIPCHK(hipDeviceSynchronize());
    clear_dgraphs(x);
    drop_derived(d);
    int rc;
    const int D = d.c.width, B = d.c.max_batch;
    d.embed = W(x, "embed");
    d.fnorm = W(x, "final.norm");
    d.pairs = W(x, "bigram");
    if ((rc = make_lin(d, d.c.untied_head ? W(x, "head") : d.embed, d.c.vocab, D, &d.head))) return rc;
    d.W.assign(d.c.n_layers, {});
    for (int i = 0; i < d.c.n_layers; ++i) {
        const pgmi_layer_spec& l = d.L[i];
        LayerW& w = d.W[i];
        for (int q = 0; q < (has_ff(l) ? 2 : 1); ++q) {
            const std::string n = std::to_string(q + 1);
            w.sub[q] = {W(x, lname(i, "hc") + n + ".in"), W(x, lname(i, "hc") + n + ".out"), W(x, lname(i, "hc") + n + ".mix"),
                        W(x, lname(i, "norm") + n)};
        }
        w.canon = W(x, lname(i, "canon1"));
        auto lin = [&](const char* name, int n, int k, Lin* o) { return make_lin(d, W(x, lname(i, name)), n, k, o); };
        if (l.mixer == PGMI_MIXER_MAMBA1) {
            if ((rc = lin("mix.in", 2 * l.inner, D, &w.in))) return rc;
            if ((rc = lin("mix.x", l.dt_rank + 2 * l.state, l.inner, &w.x))) return rc;
            if ((rc = lin("mix.dt", l.inner, l.dt_rank, &w.dt))) return rc;
            if ((rc = lin("mix.o", D, l.inner, &w.o))) return rc;
            w.conv = W(x, lname(i, "mix.conv"));
            w.conv_b = W(x, lname(i, "mix.conv.b"));
            w.dt_b = W(x, lname(i, "mix.dt.b"));
            w.A_log = W(x, lname(i, "mix.A_log"));
            w.D = W(x, lname(i, "mix.D"));
        } else if (l.mixer == PGMI_MIXER_ATTENTION) {
            if ((rc = lin("mix.q", qkv_rows(l), D, &w.in))) return rc;
            if ((rc = make_turns(d, l, &w.turns))) return rc;
            if ((rc = lin("mix.o", D, l.heads * l.vdim, &w.o))) return rc;
            w.bias = W(x, lname(i, "mix.q.b"));
            w.r1 = W(x, lname(i, "mix.r1"));
            w.r2 = W(x, lname(i, "mix.r2"));
        } else {
            if ((rc = lin("mix.z", 3 * l.width, D, &w.in))) return rc;
            if ((rc = lin("mix.o", D, l.width, &w.o))) return rc;
            uint16_t* b;  // z and x have biases, g has none
            if ((rc = derived_alloc(d, &b, (size_t)3 * l.width))) return rc;
            HIPCHK(hipMemset(b, 0, (size_t)3 * l.width * 2));
            HIPCHK(hipMemcpy(b, W(x, lname(i, "mix.z.b")), (size_t)2 * l.width * 2, hipMemcpyDeviceToDevice));
            w.bias = b;
        }
        if (l.ff) {
            if ((rc = lin("mlp.gate", 2 * l.ff, D, &w.gu))) return rc;
            if ((rc = lin("mlp.down", D, l.ff, &w.down))) return rc;
        }
        if (l.experts) {
            if ((rc = lin("mlp.e0.gate", l.experts * 2 * l.expert_ff, D, &w.egu))) return rc;
            if ((rc = lin("mlp.e0.down", l.experts * D, l.expert_ff, &w.ed))) return rc;
            if ((rc = lin("mlp.router", l.experts + l.identity + (l.shared_ff > 0), D, &w.router))) return rc;
            w.correction = W(x, lname(i, "mlp.correction"));
            if (l.shared_ff) {
                if ((rc = lin("mlp.shared.gate", 2 * l.shared_ff, D, &w.gu))) return rc;
                if ((rc = lin("mlp.shared.down", D, l.shared_ff, &w.down))) return rc;
            }
        }
    }
    LAUNCHCHK();
    if (!x->ws) {
        x->ws_bytes = (size_t)64 << 20;
        if ((rc = dalloc(x, reinterpret_cast<void**>(&x->ws), x->ws_bytes))) return rc;
        if ((rc = dalloc_t(x, &x->amax_v, (size_t)argmax_scratch_parts()))) return rc;
        if ((rc = dalloc_t(x, &x->amax_i, (size_t)argmax_scratch_parts()))) return rc;
        if ((rc = dalloc_t(x, &d.slot, (size_t)B))) return rc;
        if ((rc = dalloc_t(x, &d.pos, (size_t)B))) return rc;
        if ((rc = dalloc_t(x, &d.d_ids, (size_t)B))) return rc;
        if ((rc = dalloc_t(x, &d.d_next, (size_t)B))) return rc;
        if ((rc = dalloc_t(x, &d.pmax, (size_t)gemv_rt_parts()))) return rc;
        if ((rc = dalloc_t(x, &d.pidx, (size_t)gemv_rt_parts()))) return rc;
        HIPCHK(hipStreamCreateWithFlags(&x->cap_stream, hipStreamNonBlocking));
    }
    HIPCHK(hipDeviceSynchronize());
    d.known_slot.clear();
    x->prepared = true;
    return 0;
}

void decoder_release(pgmi_ctx* x) {
    DecoderState* d = x->dec;
    if (!d) return;
    drop_derived(*d);
    for (void* p : {d->arena, d->meta, (void*)d->part})
        if (p) (void)hipFree(p);
    delete d;
    x->dec = nullptr;
}

// Grow the workspace to these rows and chunks (captured graphs hold its addresses)
int ensure_workspace(pgmi_ctx* x, int rows, int chunks, int gchunks) {
    DecoderState& d = *x->dec;
    if (rows <= d.rows && chunks <= d.chunks && gchunks <= d.gchunks) return 0;
    rows = std::max(rows, d.rows);
    chunks = std::max(chunks, d.chunks);
    gchunks = std::max(gchunks, d.gchunks);
    HIPCHK(hipDeviceSynchronize());
    clear_dgraphs(x);
    if (d.arena) (void)hipFree(d.arena);
    d.arena = nullptr;
    d.rows = d.chunks = d.gchunks = 0;
    const int D = d.c.width;
    int l0 = r8(D), l1 = 8, l2 = 8, ldd = 8, slab_n = D, inner = 1, bcn = 2, cs = 1, cg = 1;
    int lea = 8, top = 0, ne = 0;  // mixtures: expert activations, choices per row, experts
    for (const pgmi_layer_spec& l : d.L) {
        if (l.mixer == PGMI_MIXER_MAMBA1) {
            l0 = std::max(l0, 2 * r8(l.inner));
            l1 = std::max(l1, r8(l.inner));
            l2 = std::max(l2, r8(l.inner));
            ldd = std::max(ldd, r8(l.dt_rank));
            slab_n = std::max(slab_n, l.dt_rank + 2 * l.state);
            inner = std::max(inner, l.inner);
            bcn = std::max(bcn, 2 * l.state);
            cs = std::max(cs, l.inner * l.state);
        } else if (l.mixer == PGMI_MIXER_ATTENTION) {
            l0 = std::max(l0, r8(qkv_rows(l)));
            l1 = std::max(l1, l.heads * r8(l.dim));
            l2 = std::max(l2, r8(l.heads * l.vdim));
        } else {
            l0 = std::max(l0, r8(3 * l.width));
            l2 = std::max(l2, r8(l.width));
            cg = std::max(cg, l.width);
        }
        if (const int ff = l.experts ? l.shared_ff : l.ff) {
            l2 = std::max(l2, r8(ff));
            if (d.act == ACT_F32) l0 = std::max(l0, 2 * ff);  // unfused gate|up
        }
        if (l.experts) {
            lea = std::max(lea, r8(l.expert_ff));
            top = std::max(top, l.top);
            ne = std::max(ne, l.experts);
            slab_n = std::max(slab_n, l.experts + l.identity + 1);
        }
    }
    const size_t ent = (size_t)rows * top;
    d.ldh = r8(D);
    d.ld0 = l0; d.ld1 = l1; d.ld2 = l2; d.ldd = ldd;
    d.slab_bytes = std::max<size_t>((size_t)rows * slab_n * 4, (size_t)32 << 20);
    const size_t sizes[] = {(size_t)rows * d.c.streams * D * 4, (size_t)rows * d.ldh * d.es, (size_t)rows * l0 * d.es,
                            (size_t)rows * l1 * d.es,           (size_t)rows * l2 * d.es,    (size_t)rows * ldd * d.es,
                            d.slab_bytes,                       (size_t)rows * inner * 4,    (size_t)rows * bcn * 4,
                            std::max((size_t)chunks * cs, (size_t)gchunks * 2 * cg) * 4, (size_t)chunks * inner * 4,
                            ent * lea * d.es, ent * d.ldh * d.es, ent * 4, ent * 4, (size_t)rows * 4, (size_t)rows * 4,
                            (size_t)rows * ne * 4, (size_t)(2 * ne + 2) * 4};
    constexpr int NB = sizeof(sizes) / sizeof(sizes[0]);
    size_t off[NB], total = 0;
    for (int i = 0; i < NB; ++i) {
        off[i] = total;
        total += (sizes[i] + 511) / 256 * 256;
    }
    if (hipMalloc(&d.arena, total) != hipSuccess) {
        (void)hipGetLastError();
        d.arena = nullptr;
        return fail(PGMI_E_NOMEM, "decoder workspace of " + std::to_string(total) + " bytes");
    }
    uint8_t* p = reinterpret_cast<uint8_t*>(d.arena);
    d.X = reinterpret_cast<float*>(p + off[0]);
    d.h = p + off[1]; d.p0 = p + off[2]; d.p1 = p + off[3]; d.p2 = p + off[4]; d.dtl = p + off[5];
    d.slabs = reinterpret_cast<float*>(p + off[6]);
    d.dt = reinterpret_cast<float*>(p + off[7]);
    d.bc = reinterpret_cast<float*>(p + off[8]);
    d.cstate = reinterpret_cast<float*>(p + off[9]);
    d.csum = reinterpret_cast<float*>(p + off[10]);
    d.ea = p + off[11]; d.ey = p + off[12];
    d.esel = reinterpret_cast<int*>(p + off[13]);
    d.ew = reinterpret_cast<float*>(p + off[14]);
    d.egate = reinterpret_cast<float*>(p + off[15]);
    d.inv = reinterpret_cast<float*>(p + off[16]);
    d.elist = reinterpret_cast<int*>(p + off[17]);
    d.ecnt = reinterpret_cast<int*>(p + off[18]);
    d.eactive = d.ecnt + ne;
    d.zero_words = ne + 1;
    d.rows = rows;
    d.chunks = chunks;
    d.gchunks = gchunks;
    return 0;
}

// A finished sublayer's output that the next streams pass folds in
struct Pending {
    const float* y = nullptr;
    int split = 0;
    const Sub* sub = nullptr;
    ExpertMix mix{};
};

StreamsArgs streams_args(const DecoderState& d, int rows) {
    StreamsArgs a{};
    a.X = d.X; a.rows = rows; a.S = d.c.streams; a.D = d.c.width;
    a.E = d.embed; a.escale = d.c.embed_scale; a.vocab = d.c.vocab;
    a.groups = d.c.norm_groups; a.eps = d.c.norm_eps; a.h = d.h; a.ldh = d.ldh;
    return a;
}

void fold(StreamsArgs& a, const Pending& p, int rows) {
    if (!p.y) return;
    a.y = p.y; a.ysplit = p.split; a.ystride = (long)rows * a.D;
    a.mix = p.sub->mix; a.out = p.sub->out;
}

template <typename T>
T* at(void* state, int64_t off) { return reinterpret_cast<T*>(reinterpret_cast<uint8_t*>(state) + off); }

ResidualArgs residual_args(const DecoderState& d, int rows, const Pending& p, const uint16_t* norm) {
    ResidualArgs a{};
    a.X = d.X; a.rows = rows; a.D = d.c.width; a.E = d.embed; a.escale = d.c.embed_scale; a.vocab = d.c.vocab;
    a.y = p.y; a.ysplit = p.split; a.ystride = (long)rows * a.D; a.mix = p.mix; a.mult = d.c.residual_mult;
    a.w = norm; a.w_scalar = d.c.norm_scalar; a.eps = d.c.norm_eps; a.h = d.h; a.ldh = d.ldh;
    return a;
}

// ids: the embedding makes X
void residual_embed(ResidualArgs& a, const DecoderState& d, const int64_t* ids, void* state, const StateMap& st, int max_tokens) {
    a.ids = ids;
    if (!d.c.bigram_buckets) return;
    a.pairs = d.pairs; a.mul_prev = d.c.bigram_mul_prev; a.mul_cur = d.c.bigram_mul_cur; a.buckets = d.c.bigram_buckets;
    a.history = reinterpret_cast<int*>(reinterpret_cast<uint8_t*>(state) + st.history);
    a.max_tokens = max_tokens;
}

WAttnHeads attn_heads(const DecoderState& d, const pgmi_layer_spec& l, const LayerW& w) {
    return {l.heads, l.kv_heads, l.dim, l.vdim, r8(l.dim), r8(l.vdim), l.kv_from < 0, l.qk_norm != 0, l.v_norm != 0,
            d.c.norm_eps, w.turns, l.rot_dims};
}
WAttnScore attn_score(const pgmi_layer_spec& l, const LayerW& w) {
    return {l.window, l.keep_first, l.scale, l.softcap, w.r1, w.r2};
}

RouteArgs route_args(const DecoderState& d, const pgmi_layer_spec& l, const LayerW& w, int rows, int split) {
    RouteArgs a{};
    a.z = d.slabs; a.split = split; a.ldz = w.router.n; a.zstride = (long)rows * a.ldz; a.rows = rows;
    a.n = l.experts + l.identity; a.experts = l.experts; a.top = l.top; a.groups = l.groups; a.keep = l.groups_keep;
    a.correction = w.correction; a.sel = d.esel; a.w = d.ew; a.gate = l.shared_ff ? d.egate : nullptr;
    a.cnt = d.ecnt; a.list = d.elist; a.cap = rows;
    return a;
}
ExpertArgs expert_args(const DecoderState& d, const pgmi_layer_spec& l, const LayerW& w, int rows, ExpertMode mode) {
    ExpertArgs a{};
    const bool up = mode == EX_SWIGLU;
    const Lin& lin = up ? w.egu : w.ed;
    a.A = up ? d.h : d.ea; a.lda = up ? d.ldh : r8(l.expert_ff); a.gather = up ? l.top : 1;
    a.W = lin.w; a.ldw = lin.ldw; a.K = lin.k; a.N = up ? l.expert_ff : d.c.width;
    a.wstride = (long)(up ? 2 : 1) * a.N * lin.ldw;
    a.out = up ? d.ea : d.ey; a.ldo = up ? r8(l.expert_ff) : d.ldh;
    a.cnt = d.ecnt; a.list = d.elist; a.cap = rows; a.experts = l.experts; a.entries = rows * l.top;
    return a;
}
ExpertMix expert_mix(const DecoderState& d, const pgmi_layer_spec& l) {
    return {d.ey, d.ldh, d.esel, d.ew, l.top, l.experts, d.h, d.ldh, l.shared_ff ? d.egate : nullptr};
}

// device addresses of a step's metadata
struct Meta {
    const SeqInfo* seqs;
    int nseq;
    struct Chunks {
        const ChunkInfo* p;
        int n;
        bool multi;  // some sequence has more than one
    } scan, gru;
    const int* row_seq;
    const int* want;
    std::map<int, std::pair<const ChunkInfo*, int>> tiles;  // by query heads per key/value head
};

int forward_body(pgmi_ctx* x, hipStream_t s, const int64_t* ids, int rows, const Meta& m, void* state, int n_slots,
                 int max_tokens, int n_want, float* logits, float* taps) {
    DecoderState& d = *x->dec;
    const int D = d.c.width;
    const StateMap sm = state_layout(d, n_slots, max_tokens);
    const std::vector<StateAt>& st = sm.at;
    Pending pend;
    bool first = true;
    // the finished sublayer folded into the residual, and the input of sublayer q of layer i in d.h
    auto read = [&](int i, int q, float* tap) {
        const LayerW& w = d.W[i];
        const Sub& sub = w.sub[q];
        if (d.c.plain_residual) {
            ResidualArgs a = residual_args(d, rows, pend, sub.norm);
            const bool conv = q == 0 && d.c.canon_taps > 0;
            if (first) residual_embed(a, d, ids, state, sm, max_tokens);
            a.seqs = m.seqs; a.row_seq = m.row_seq; a.tap = tap;
            if (conv) { a.h = nullptr; a.inv = d.inv; }
            if (q == 1 && d.L[i].experts) { a.zero = d.ecnt; a.nzero = d.L[i].experts; }
            residual_norm(s, d.act, a);
            if (conv) {
                CanonArgs c{};
                c.X = d.X; c.inv = d.inv; c.w = sub.norm; c.w_scalar = d.c.norm_scalar; c.rows = rows; c.D = D;
                c.taps = d.c.canon_taps; c.cw = w.canon; c.ring = at<float>(state, st[i].ring); c.h = d.h; c.ldh = d.ldh;
                c.seqs = m.seqs; c.nseq = m.nseq; c.chunks = m.scan.p; c.nchunk = m.scan.n;
                canon(s, d.act, c);
            }
            pend = {};
            first = false;
            return;
        }
        StreamsArgs a = streams_args(d, rows);
        if (first) a.ids = ids;
        fold(a, pend, rows);
        a.in = sub.in; a.w = sub.norm; a.tap = tap;
        streams_norm(s, d.act, a);
        pend = {};
        first = false;
    };
    auto out_proj = [&](const Lin& o, const void* in, int ldin, const Sub& sub) {
        pend.split = matmul_rt(s, d.act, in, ldin, o.w, o.ldw, rows, D, o.k, RT_SLABS, nullptr, d.slabs, D, d.slab_bytes, nullptr);
        pend.y = d.slabs;
        pend.sub = &sub;
    };
    for (int i = 0; i < d.c.n_layers; ++i) {
        const pgmi_layer_spec& l = d.L[i];
        const LayerW& w = d.W[i];
        read(i, 0, taps && i ? taps + (long)(i - 1) * rows * D : nullptr);
        if (l.mixer == PGMI_MIXER_MAMBA1) {
            const int C = l.inner, N = l.state, R = l.dt_rank, ldc = r8(C), ldxz = r8(2 * C), ldd = r8(R);
            matmul_rt(s, d.act, d.h, d.ldh, w.in.w, w.in.ldw, rows, 2 * C, w.in.k, RT_ACT, nullptr, d.p0, ldxz, 0, nullptr);
            conv_silu(s, d.act, d.p0, ldxz, C, l.conv, w.conv, w.conv_b, m.seqs, m.nseq, m.scan.p, m.scan.n,
                      at<float>(state, st[i].a), d.p1, ldc);
            const int sp = matmul_rt(s, d.act, d.p1, ldc, w.x.w, w.x.ldw, rows, R + 2 * N, w.x.k, RT_SLABS, nullptr, d.slabs,
                                     0, d.slab_bytes, nullptr);
            scan_inputs(s, d.act, d.slabs, sp, rows, R, N, d.dtl, ldd, d.bc);
            matmul_rt(s, d.act, d.dtl, ldd, w.dt.w, w.dt.ldw, rows, C, w.dt.k, RT_F32, nullptr, d.dt, C, 0, nullptr);
            ScanArgs a{};
            a.dt = d.dt; a.dtb = w.dt_b; a.x = d.p1; a.ldx = ldc; a.z = d.p0 + (size_t)C * d.es; a.ldz = ldxz; a.bc = d.bc;
            a.A_log = w.A_log; a.Dw = w.D; a.state = at<float>(state, st[i].b); a.cstate = d.cstate; a.csum = d.csum;
            a.y = d.p2; a.ldy = ldc; a.C = C; a.N = N; a.seqs = m.seqs; a.nseq = m.nseq; a.chunks = m.scan.p;
            a.nchunk = m.scan.n; a.multi = m.scan.multi;
            selective_scan(s, d.act, a);
            out_proj(w.o, d.p2, ldc, w.sub[0]);
        } else if (l.mixer == PGMI_MIXER_ATTENTION) {
            WAttnArgs a{};
            a.hd = attn_heads(d, l, w); a.sc = attn_score(l, w);
            a.ldqkv = r8(w.in.n); a.ldo = r8(l.heads * l.vdim);
            matmul_rt(s, d.act, d.h, d.ldh, w.in.w, w.in.ldw, rows, w.in.n, w.in.k, RT_ACT, w.bias, d.p0, a.ldqkv, 0, nullptr);
            a.qkv = d.p0; a.q = d.p1; a.kc = at<void>(state, st[i].a); a.vc = at<void>(state, st[i].b);
            a.max_tokens = max_tokens; a.o = d.p2; a.rows = rows; a.seqs = m.seqs; a.nseq = m.nseq; a.row_seq = m.row_seq;
            const auto& t = m.tiles.at(l.heads / l.kv_heads);
            a.tiles = t.first; a.ntile = t.second;
            wattn_append(s, d.act, a);
            wattn_prefill(s, d.act, a);
            out_proj(w.o, d.p2, a.ldo, w.sub[0]);
        } else {
            const int C = l.width, ldz = r8(3 * C), ldc = r8(C);
            matmul_rt(s, d.act, d.h, d.ldh, w.in.w, w.in.ldw, rows, 3 * C, w.in.k, RT_ACT, w.bias, d.p0, ldz, 0, nullptr);
            GruArgs a{};
            a.zug = d.p0; a.ld = ldz; a.state = at<float>(state, st[i].a); a.cstate = d.cstate; a.y = d.p2; a.ldy = ldc;
            a.C = C; a.seqs = m.seqs; a.nseq = m.nseq; a.chunks = m.gru.p; a.nchunk = m.gru.n; a.multi = m.gru.multi;
            mingru_scan(s, d.act, a);
            out_proj(w.o, d.p2, ldc, w.sub[0]);
        }
        if (has_ff(l)) read(i, 1, nullptr);
        if (l.experts) {
            const int sp = matmul_rt(s, d.act, d.h, d.ldh, w.router.w, w.router.ldw, rows, w.router.n, w.router.k, RT_SLABS,
                                     nullptr, d.slabs, 0, d.slab_bytes, nullptr);
            route(s, route_args(d, l, w, rows, sp));
            experts_rt(s, d.act, EX_SWIGLU, expert_args(d, l, w, rows, EX_SWIGLU));
            experts_rt(s, d.act, EX_STORE, expert_args(d, l, w, rows, EX_STORE));
        }
        if (const int ff = l.experts ? l.shared_ff : l.ff) {
            matmul_rt(s, d.act, d.h, d.ldh, w.gu.w, w.gu.ldw, rows, ff, w.gu.k, RT_SWIGLU, nullptr, d.p2, r8(ff), 0,
                      reinterpret_cast<float*>(d.p0));
            out_proj(w.down, d.p2, r8(ff), w.sub[1]);
        }
        if (l.experts) pend.mix = expert_mix(d, l);
    }
    if (taps && d.c.plain_residual) {
        ResidualArgs a = residual_args(d, rows, pend, nullptr);
        a.h = nullptr;
        a.tap = taps + (long)(d.c.n_layers - 1) * rows * D;
        residual_norm(s, d.act, a);
        pend = {};
    } else if (taps) {
        StreamsArgs a = streams_args(d, rows);
        fold(a, pend, rows);
        a.h = nullptr;
        a.tap = taps + (long)(d.c.n_layers - 1) * rows * D;
        streams_norm(s, d.act, a);
        pend = {};
    }
    if (n_want > 0) {
        const void* h = d.h;
        if (d.c.plain_residual) {
            ResidualArgs a = residual_args(d, rows, pend, d.fnorm);
            a.rows = n_want; a.rows_idx = m.want;
            h = a.h = d.p0;  // other rows' d.h is still read (identity experts)
            residual_norm(s, d.act, a);
        } else {
            StreamsArgs a = streams_args(d, n_want);
            fold(a, pend, rows);
            a.in = nullptr; a.w = d.fnorm; a.rows_idx = m.want;
            streams_norm(s, d.act, a);
        }
        const GemvRtForm form = gemv_rt_form(n_want, d.act, 1, 1);
        if (gemv_rt_fits(form, d.head.k, d.act)) {
            GemvRtArgs g{};
            g.form = form; g.B = n_want; g.N = d.c.vocab; g.K = d.head.k; g.W = d.head.w; g.ldw = d.head.ldw; g.x = h; g.ldx = d.ldh;
            g.out = logits; g.ldo = d.c.vocab;
            gemv_rt(s, d.act, GR_F32, g);
        } else {
            matmul_rt(s, d.act, h, d.ldh, d.head.w, d.head.ldw, n_want, d.c.vocab, d.head.k, RT_F32, nullptr, logits,
                      d.c.vocab, 0, nullptr);
        }
    }
    LAUNCHCHK();
    return 0;
}

int decode_body_rt(pgmi_ctx* x, hipStream_t s, const int64_t* ids, int B, void* state, int n_slots, int max_tokens,
                   float* logits, int64_t* next, int64_t* hist) {
    DecoderState& d = *x->dec;
    const int D = d.c.width, V = d.c.vocab;
    const StateMap sm = state_layout(d, n_slots, max_tokens);
    const std::vector<StateAt>& st = sm.at;
    const bool plain = d.c.plain_residual;
    if (!plain) {  // the embedding rows into every stream, and the first sublayer's input
        StreamsArgs a = streams_args(d, B);
        a.ids = ids; a.in = d.W[0].sub[0].in; a.w = d.W[0].sub[0].norm;
        streams_norm(s, d.act, a);
    }
    const GemvRtForm form = gemv_rt_form(B, d.act, d.c.streams, D);
    bool have_h = !plain;  // d.h holds the coming sublayer's input
    bool first = true;     // plain residual: X is not made yet
    Pending pend;
    // plain residual: the finished sublayer folded in and the input of sublayer q of layer i (the end: i = n_layers) in d.h;
    // router: a mixture's choice in the same launch
    auto read = [&](int i, int q, const RouteArgs* router = nullptr) {
        if (!plain) return;
        const bool end = i == d.c.n_layers;
        ResidualArgs a = residual_args(d, B, pend, end ? d.fnorm : d.W[i].sub[q].norm);
        if (first) residual_embed(a, d, ids, state, sm, max_tokens);
        a.slot = d.slot; a.pos = d.pos;
        if (!end && q == 0 && d.c.canon_taps > 0) {
            a.taps = d.c.canon_taps; a.cw = d.W[i].canon; a.ring = at<float>(state, st[i].ring);
        }
        if (!end && q == 0 && d.L[i].experts) { a.zero = d.ecnt; a.nzero = d.zero_words; }
        if (router) residual_route(s, a, d.W[i].router.w, d.W[i].router.ldw, *router);
        else residual_norm(s, d.act, a);
        pend = {};
        first = false;
        have_h = true;
    };
    // the input side of a projection: d.h, or (fused) the streams' read and norm inside the GEMV
    auto base = [&](const Sub& sub, const Lin& w, bool fused) {
        if (!have_h && (!fused || pend.y || form != GF_STREAM)) {
            StreamsArgs a = streams_args(d, B);
            fold(a, pend, B);
            a.in = sub.in; a.w = sub.norm;
            streams_norm(s, d.act, a);
            pend = {};
            have_h = true;
        }
        GemvRtArgs g{};
        g.form = form; g.B = B; g.N = w.n; g.K = w.k; g.W = w.w; g.ldw = w.ldw; g.S = d.c.streams; g.D = D; g.groups = d.c.norm_groups;
        g.eps = d.c.norm_eps; g.X = d.X; g.in = sub.in; g.nw = sub.norm; g.slot = d.slot; g.pos = d.pos;
        if (have_h) { g.x = d.h; g.ldx = d.ldh; }
        have_h = false;
        return g;
    };
    auto row_in = [&](const Lin& w, const void* in, int ldin) {
        GemvRtArgs g{};
        g.form = form; g.B = B; g.N = w.n; g.K = w.k; g.W = w.w; g.ldw = w.ldw; g.x = in; g.ldx = ldin; g.slot = d.slot; g.pos = d.pos;
        return g;
    };
    auto out_proj = [&](const Lin& o, const void* in, int ldin, const Sub& sub) {
        const bool fits = gemv_rt_fits(form, o.k, d.act);
        if (fits && form != GF_STREAM) {  // the next streams pass sums the slabs
            GemvRtArgs g = row_in(o, in, ldin);
            g.out = d.slabs; g.ldo = D; g.split = gemv_rt_split(form, D, o.k);
            gemv_rt(s, d.act, GR_F32, g);
            pend = {d.slabs, g.split, &sub, {}};
        } else if (fits) {
            GemvRtArgs g = row_in(o, in, ldin);
            g.X = d.X; g.S = d.c.streams; g.D = D; g.mix = sub.mix; g.wout = sub.out; g.mult = d.c.residual_mult;
            gemv_rt(s, d.act, GR_STREAMS, g);
        } else {
            pend.split = matmul_rt(s, d.act, in, ldin, o.w, o.ldw, B, D, o.k, RT_SLABS, nullptr, d.slabs, D, d.slab_bytes, nullptr);
            pend.y = d.slabs;
            pend.sub = &sub;
        }
    };
    for (int i = 0; i < d.c.n_layers; ++i) {
        const pgmi_layer_spec& l = d.L[i];
        const LayerW& w = d.W[i];
        const bool fin = gemv_rt_fits(form, w.in.k, d.act);
        read(i, 0);
        if (l.mixer == PGMI_MIXER_MAMBA1) {
            const int C = l.inner, N = l.state, R = l.dt_rank, ldc = r8(C);
            float* taps = at<float>(state, st[i].a);
            ScanStepArgs a{};
            GemvRtArgs g = base(w.sub[0], w.in, fin);
            if (fin) {
                g.out = d.p1; g.ldo = ldc; g.out2 = d.p0; g.ldo2 = ldc; g.C = C; g.taps_k = l.conv; g.cw = w.conv;
                g.cb = w.conv_b; g.state = taps;
                gemv_rt(s, d.act, GR_CONV, g);
                a.z = d.p0; a.ldz = ldc;
            } else {
                const int ldxz = r8(2 * C);
                matmul_rt(s, d.act, d.h, d.ldh, w.in.w, w.in.ldw, B, 2 * C, w.in.k, RT_ACT, nullptr, d.p0, ldxz, 0, nullptr);
                conv_step(s, d.act, d.p0, ldxz, B, C, l.conv, w.conv, w.conv_b, taps, d.slot, d.pos, d.p1, ldc);
                a.z = d.p0 + (size_t)C * d.es; a.ldz = ldxz;
            }
            a.split = 1;
            if (gemv_rt_fits(form, w.x.k, d.act)) {
                g = row_in(w.x, d.p1, ldc);
                g.out = d.slabs; g.ldo = w.x.n; g.split = gemv_rt_split(form, w.x.n, w.x.k);
                gemv_rt(s, d.act, GR_F32, g);
                a.split = g.split;
            } else {
                a.split = matmul_rt(s, d.act, d.p1, ldc, w.x.w, w.x.ldw, B, w.x.n, w.x.k, RT_SLABS, nullptr, d.slabs, 0,
                                    d.slab_bytes, nullptr);
            }
            a.slabs = d.slabs; a.Wdt = w.dt.w; a.ldwdt = w.dt.ldw; a.dtb = w.dt_b; a.x = d.p1; a.ldx = ldc; a.A_log = w.A_log;
            a.Dw = w.D; a.state = at<float>(state, st[i].b); a.slot = d.slot; a.pos = d.pos; a.y = d.p2; a.ldy = ldc;
            a.B = B; a.C = C; a.N = N; a.R = R;
            scan_step(s, d.act, a);
            out_proj(w.o, d.p2, ldc, w.sub[0]);
        } else if (l.mixer == PGMI_MIXER_ATTENTION) {
            WAttnDecodeArgs a{};
            a.hd = attn_heads(d, l, w); a.sc = attn_score(l, w);
            a.ldqkv = r8(w.in.n); a.ldo = r8(l.heads * l.vdim);
            GemvRtArgs g = base(w.sub[0], w.in, fin);
            if (fin) {
                g.out = d.p0; g.ldo = a.ldqkv; g.bias = w.bias;
                gemv_rt(s, d.act, GR_ACT, g);
            } else {
                matmul_rt(s, d.act, d.h, d.ldh, w.in.w, w.in.ldw, B, w.in.n, w.in.k, RT_ACT, w.bias, d.p0, a.ldqkv, 0, nullptr);
            }
            a.qkv = d.p0; a.kc = at<void>(state, st[i].a); a.vc = at<void>(state, st[i].b); a.max_tokens = max_tokens;
            a.o = d.p2; a.B = B; a.slot = d.slot; a.pos = d.pos; a.part = d.part;
            a.nsplit = wattn_decode_splits(B, l.kv_heads, a.sc, max_tokens);
            wattn_decode(s, d.act, a);
            out_proj(w.o, d.p2, a.ldo, w.sub[0]);
        } else {
            const int C = l.width, ldc = r8(C);
            GemvRtArgs g = base(w.sub[0], w.in, fin);
            if (fin) {
                g.N = C; g.out = d.p2; g.ldo = ldc; g.bias = w.bias; g.state = at<float>(state, st[i].a);
                gemv_rt(s, d.act, GR_GRU, g);
            } else {
                matmul_rt(s, d.act, d.h, d.ldh, w.in.w, w.in.ldw, B, 3 * C, w.in.k, RT_ACT, w.bias, d.p0, r8(3 * C), 0, nullptr);
                gru_step(s, d.act, d.p0, r8(3 * C), B, C, at<float>(state, st[i].a), d.slot, d.pos, d.p2, ldc);
            }
            out_proj(w.o, d.p2, ldc, w.sub[0]);
        }
        const bool few = l.experts && residual_route_fits(d.act, B, D);
        if (has_ff(l) && !few) read(i, 1);
        if (few) {  // router and choice behind the norm; the shared expert rides along with the others
            RouteArgs r = route_args(d, l, w, B, 1);
            r.active = d.eactive;
            read(i, 1, &r);
            ExpertArgs up = expert_args(d, l, w, B, EX_SWIGLU), down = expert_args(d, l, w, B, EX_STORE);
            up.active = down.active = d.eactive;
            up.B = down.B = B;
            if (l.shared_ff) {
                up.Wsh = w.gu.w; up.ldwsh = w.gu.ldw; up.Nsh = l.shared_ff; up.Ksh = w.gu.k; up.Ash = d.h; up.ldash = d.ldh;
                up.outsh = d.p2; up.ldosh = r8(l.shared_ff);
                down.Wsh = w.down.w; down.ldwsh = w.down.ldw; down.Nsh = D; down.Ksh = w.down.k; down.Ash = d.p2;
                down.ldash = r8(l.shared_ff); down.outsh = d.slabs; down.ldosh = D;
            }
            experts_skinny(s, EX_SWIGLU, up);
            experts_skinny(s, EX_STORE, down);
            if (l.shared_ff) pend = {d.slabs, 1, &w.sub[1], {}};
        } else if (l.experts) {
            const bool fr = gemv_rt_fits(form, w.router.k, d.act);
            GemvRtArgs g = base(w.sub[1], w.router, fr);
            int sp;
            if (fr) {
                g.out = d.slabs; g.ldo = w.router.n; sp = g.split = gemv_rt_split(form, w.router.n, w.router.k);
                gemv_rt(s, d.act, GR_F32, g);
            } else {
                sp = matmul_rt(s, d.act, d.h, d.ldh, w.router.w, w.router.ldw, B, w.router.n, w.router.k, RT_SLABS, nullptr,
                               d.slabs, 0, d.slab_bytes, nullptr);
            }
            route(s, route_args(d, l, w, B, sp));
            experts_rt(s, d.act, EX_SWIGLU, expert_args(d, l, w, B, EX_SWIGLU));
            experts_rt(s, d.act, EX_STORE, expert_args(d, l, w, B, EX_STORE));
        }
        if (const int ff = few ? 0 : l.experts ? l.shared_ff : l.ff) {
            const bool fgu = gemv_rt_fits(form, w.gu.k, d.act);
            if (l.experts) have_h = true;  // the mixture's input, once more
            GemvRtArgs g = base(w.sub[1], w.gu, fgu);
            if (fgu) {
                g.N = ff; g.out = d.p2; g.ldo = r8(ff);
                gemv_rt(s, d.act, GR_SWIGLU, g);
            } else {
                matmul_rt(s, d.act, d.h, d.ldh, w.gu.w, w.gu.ldw, B, ff, w.gu.k, RT_SWIGLU, nullptr, d.p2, r8(ff), 0,
                          reinterpret_cast<float*>(d.p0));
            }
            if (l.experts) {  // the next residual pass scales it by its gate
                pend.split = matmul_rt(s, d.act, d.p2, r8(ff), w.down.w, w.down.ldw, B, D, w.down.k, RT_SLABS, nullptr, d.slabs, D,
                                       d.slab_bytes, nullptr);
                pend.y = d.slabs;
            } else {
                out_proj(w.down, d.p2, r8(ff), w.sub[1]);
            }
        }
        if (l.experts) pend.mix = expert_mix(d, l);
    }
    read(d.c.n_layers, 0);
    const Sub fin{nullptr, nullptr, nullptr, d.fnorm};
    const bool fl = gemv_rt_fits(form, d.head.k, d.act);
    GemvRtArgs g = base(fin, d.head, fl);
    if (fl) {
        g.out = logits; g.ldo = V; g.pmax = d.pmax; g.pidx = d.pidx;
        gemv_rt(s, d.act, GR_LOGITS, g);
        const int parts = form == GF_STREAM ? gemv_rt_blocks(g, GR_LOGITS) : 0;
        if (!parts) argmax_rows(s, logits, B, V, x->amax_v, x->amax_i, next);
        decode_finish(s, B, d.pmax, d.pidx, parts, next, hist, d.pos);
    } else {
        matmul_rt(s, d.act, d.h, d.ldh, d.head.w, d.head.ldw, B, V, d.head.k, RT_F32, nullptr, logits, V, 0, nullptr);
        argmax_rows(s, logits, B, V, x->amax_v, x->amax_i, next);
        decode_finish(s, B, nullptr, nullptr, 0, next, hist, d.pos);
    }
    return 0;
}

int check_state(const DecoderState& d, void* state, int n_slots, int max_tokens) {
    if (!state) return fail(PGMI_E_ARG, "null state");
    if (reinterpret_cast<uintptr_t>(state) % 256 != 0) return fail(PGMI_E_ARG, "the state slab must be 256-byte aligned");
    if (n_slots < 1 || max_tokens < 1) return fail(PGMI_E_ARG, "empty state");
    (void)d;
    return 0;
}

int check_seqs(const DecoderState& d, int n, const int32_t* slots, int n_slots) {
    if (n < 1 || n > d.c.max_batch) return fail(PGMI_E_ARG, "batch exceeds max_batch");
    std::set<int> seen;
    for (int r = 0; r < n; ++r) {
        if (slots[r] < 0 || slots[r] >= n_slots) return fail(PGMI_E_ARG, "slot out of range");
        if (!seen.insert(slots[r]).second) return fail(PGMI_E_ARG, "a slot appears twice in one step");
    }
    return 0;
}

}  // namespace

extern "C" {

int pgmi_decoder_create(int device, const pgmi_decoder_config* cfg, const pgmi_layer_spec* layers, pgmi_ctx** out) {
    if (!cfg || !layers || !out) return fail(PGMI_E_ARG, "null argument");
    const pgmi_decoder_config& c = *cfg;
    if (c.vocab < 1 || c.width < 1 || c.n_layers < 1) return fail(PGMI_E_ARG, "vocab, width and layers must be positive");
    if (c.streams < 1 || c.streams > 8) return fail(PGMI_E_ARG, "streams must be in [1, 8]");
    if (c.norm_groups < 1 || c.width % c.norm_groups != 0) return fail(PGMI_E_ARG, "norm groups must divide the width");
    if (c.plain_residual && (c.streams != 1 || c.norm_groups != 1))
        return fail(PGMI_E_ARG, "a plain residual has one stream and one norm group");
    if (!c.plain_residual && (c.norm_scalar || c.canon_taps || c.bigram_buckets))
        return fail(PGMI_E_ARG, "scalar norms, the input convolution and token pairs go with a plain residual");
    if (c.canon_taps < 0 || c.bigram_buckets < 0) return fail(PGMI_E_ARG, "negative taps or buckets");
    if (c.bigram_buckets && (c.bigram_mul_prev < 0 || c.bigram_mul_cur < 0 || c.bigram_mul_prev >= c.bigram_buckets ||
                             c.bigram_mul_cur >= c.bigram_buckets))
        return fail(PGMI_E_ARG, "token pair factors must be reduced modulo the buckets");
    if (c.width > 16384) return fail(PGMI_E_ARG, "width must be at most 16384");
    if (c.max_batch < 1) return fail(PGMI_E_ARG, "max_batch must be positive");
    if (c.act_dtype != PGMI_DTYPE_BF16 && c.act_dtype != PGMI_DTYPE_F32)
        return fail(PGMI_E_ARG, "activations are bf16 or fp32");
    for (int i = 0; i < c.n_layers; ++i) {
        const pgmi_layer_spec& l = layers[i];
        const std::string at = "layer " + std::to_string(i) + ": ";
        if (l.ff < 0) return fail(PGMI_E_ARG, at + "negative feed-forward size");
        if (l.mixer == PGMI_MIXER_MAMBA1) {
            if (l.conv < 1 || l.dt_rank < 1 || l.inner < 1 || l.state < 1) return fail(PGMI_E_ARG, at + "mamba1 sizes must be positive");
            if (l.state > scan_max_state()) return fail(PGMI_E_ARG, at + "at most 256 states per channel");
        } else if (l.mixer == PGMI_MIXER_ATTENTION) {
            if (l.heads < 1 || l.kv_heads < 1 || l.dim < 1 || l.vdim < 1 || l.window < 1)
                return fail(PGMI_E_ARG, at + "attention sizes must be positive");
            if (l.heads % l.kv_heads != 0) return fail(PGMI_E_ARG, at + "kv_heads must divide heads");
            if (l.dim > 512 || l.vdim > 2048) return fail(PGMI_E_ARG, at + "head sizes are at most 512 (query / key) and 2048 (value)");
            if (l.keep_first < 0) return fail(PGMI_E_ARG, at + "negative number of kept tokens");
            if (l.softcap < 0 || (l.softcap > 0 && l.distance_bias))
                return fail(PGMI_E_ARG, at + "the score cap must be positive, and goes without a distance bias");
            if (l.rot_dims < 0 || l.rot_dims % 2 != 0 || l.rot_dims > l.dim || (l.rot_dims > 0 && !(l.rot_base > 0)))
                return fail(PGMI_E_ARG, at + "rotated dims must be even and inside the head, with a positive base");
            if (l.rot_original > 0 && !(l.rot_factor > 0 && l.rot_low > 0 && l.rot_high > l.rot_low))
                return fail(PGMI_E_ARG, at + "rotary scaling needs a factor and 0 < low < high");
            if (l.kv_from >= i) return fail(PGMI_E_ARG, at + "keys and values come from an earlier layer");
            if (l.kv_from >= 0) {
                const pgmi_layer_spec& k = layers[l.kv_from];
                if (k.mixer != PGMI_MIXER_ATTENTION || k.kv_from >= 0 || k.kv_heads != l.kv_heads || k.dim != l.dim || k.vdim != l.vdim)
                    return fail(PGMI_E_ARG, at + "keys and values come from an attention layer with its own, of equal sizes");
            }
        } else if (l.mixer == PGMI_MIXER_MINGRU) {
            if (l.width < 1) return fail(PGMI_E_ARG, at + "mingru width must be positive");
        } else {
            return fail(PGMI_E_ARG, at + "unknown mixer");
        }
        if (l.experts < 0 || l.identity < 0 || l.shared_ff < 0) return fail(PGMI_E_ARG, at + "negative expert sizes");
        if (l.experts) {
            const int n = l.experts + l.identity;
            if (!c.plain_residual) return fail(PGMI_E_ARG, at + "a mixture of experts goes with a plain residual");
            if (l.ff) return fail(PGMI_E_ARG, at + "a feed-forward is gated or a mixture of experts");
            if (n > kMaxExperts) return fail(PGMI_E_ARG, at + "at most " + std::to_string(kMaxExperts) + " experts");
            if (l.expert_ff < 1) return fail(PGMI_E_ARG, at + "expert size must be positive");
            if (l.groups < 1 || n % l.groups != 0 || l.groups_keep < 1 || l.groups_keep > l.groups)
                return fail(PGMI_E_ARG, at + "groups must divide the experts, and some of them be kept");
            if (l.top < 1 || l.top > n / l.groups * l.groups_keep)
                return fail(PGMI_E_ARG, at + "more experts per token than the kept groups hold");
        }
    }
    auto* x = new pgmi_ctx();
    x->family = FAMILY_DECODER;
    x->device = device;
    x->prepare = decoder_prepare;
    x->kv_bytes = decoder_state_bytes;
    x->release = decoder_release;
    x->dec = new DecoderState();
    x->dec->c = c;
    x->dec->L.assign(layers, layers + c.n_layers);
    x->dec->act = c.act_dtype == PGMI_DTYPE_F32 ? ACT_F32 : ACT_BF16;
    x->dec->es = c.act_dtype == PGMI_DTYPE_F32 ? 4 : 2;
    build_decoder_layout(x);
    *out = x;
    return 0;
}

int pgmi_decoder_forward(pgmi_ctx* x, const int64_t* ids, int n_seq, const int32_t* slots, const int32_t* starts,
                         const int32_t* lens, void* state, int n_slots, int max_tokens, const int32_t* want, int n_want,
                         float* logits, float* taps, void* stream) {
    int rc;
    if ((rc = ensure_prepared(x, FAMILY_DECODER))) return rc;
    DecoderState& d = *x->dec;
    if (!ids || !slots || !starts || !lens || n_want < 0 || (n_want > 0 && (!want || !logits)))
        return fail(PGMI_E_ARG, "null argument");
    if ((rc = check_state(d, state, n_slots, max_tokens)) || (rc = check_seqs(d, n_seq, slots, n_slots))) return rc;
    long total = 0;
    for (int r = 0; r < n_seq; ++r) {
        if (lens[r] < 1) return fail(PGMI_E_ARG, "every sequence brings at least one token");
        if (starts[r] < 0 || (long)starts[r] + lens[r] > max_tokens) return fail(PGMI_E_ARG, "state capacity exceeded");
        total += lens[r];
    }
    if (total > (1 << 24)) return fail(PGMI_E_ARG, "too many tokens in one step");
    const int rows = (int)total;
    for (int i = 0; i < n_want; ++i)
        if (want[i] < 0 || want[i] >= rows) return fail(PGMI_E_ARG, "wanted row out of range");
    HIPCHK(hipSetDevice(x->device));
    hipStream_t s = (hipStream_t)stream;
    // metadata: sequences, scan chunks, attention tiles per head grouping, row -> sequence, wanted rows
    std::vector<int>& m = d.host;
    m.clear();
    auto put = [&](std::initializer_list<int> v) { m.insert(m.end(), v); };
    for (int r = 0, off = 0; r < n_seq; off += lens[r], ++r) put({off, lens[r], starts[r], slots[r]});
    struct Cut { size_t o; int n; bool multi; };
    auto cut = [&](int ct) {
        Cut c{m.size(), 0, false};
        for (int r = 0, off = 0; r < n_seq; off += lens[r], ++r) {
            const int n = (lens[r] + ct - 1) / ct;
            c.multi |= n > 1;
            for (int k = 0; k < n; ++k, ++c.n) put({r, off + k * ct, std::min(ct, lens[r] - k * ct), k * ct, k, n});
        }
        return c;
    };
    const Cut scan = cut(rows <= 16384 ? 64 : 256), gru = cut(rows <= 16384 ? 32 : 128);
    struct Tiles { int R; size_t o; int n; };
    std::vector<Tiles> tiles;
    for (const pgmi_layer_spec& l : d.L) {
        if (l.mixer != PGMI_MIXER_ATTENTION) continue;
        const int R = l.heads / l.kv_heads;
        if (std::any_of(tiles.begin(), tiles.end(), [&](const Tiles& t) { return t.R == R; })) continue;
        Tiles t{R, m.size(), 0};
        for (int r = 0; r < n_seq; ++r) {
            if ((long)lens[r] * R > INT32_MAX - kWAttnRows) return fail(PGMI_E_ARG, "too many tokens in one step");
            for (int f = 0; f < lens[r] * R; f += kWAttnRows, ++t.n) put({r, 0, kWAttnRows, f, 0, 0});
        }
        tiles.push_back(t);
    }
    const size_t o_row = m.size();
    for (int r = 0; r < n_seq; ++r) m.insert(m.end(), lens[r], r);
    const size_t o_want = m.size();
    m.insert(m.end(), want, want + n_want);
    if ((rc = ensure_workspace(x, std::max(rows, n_want), scan.n, gru.n))) return rc;
    if (m.size() * 4 > d.meta_bytes) {
        HIPCHK(hipDeviceSynchronize());
        if (d.meta) (void)hipFree(d.meta);
        d.meta = nullptr;
        d.meta_bytes = 0;
        const size_t nb = m.size() * 4 * 2;
        if (hipMalloc(&d.meta, nb) != hipSuccess) {
            d.meta = nullptr;
            return fail(PGMI_E_NOMEM, "step metadata");
        }
        d.meta_bytes = nb;
    }
    HIPCHK(hipMemcpyAsync(d.meta, m.data(), m.size() * 4, hipMemcpyHostToDevice, s));
    const int* dm = reinterpret_cast<const int*>(d.meta);
    Meta meta{};
    meta.seqs = reinterpret_cast<const SeqInfo*>(dm);
    meta.nseq = n_seq;
    meta.scan = {reinterpret_cast<const ChunkInfo*>(dm + scan.o), scan.n, scan.multi};
    meta.gru = {reinterpret_cast<const ChunkInfo*>(dm + gru.o), gru.n, gru.multi};
    meta.row_seq = dm + o_row;
    meta.want = dm + o_want;
    for (const Tiles& t : tiles) meta.tiles[t.R] = {reinterpret_cast<const ChunkInfo*>(dm + t.o), t.n};
    return forward_body(x, s, ids, rows, meta, state, n_slots, max_tokens, n_want, logits, taps);
}

int pgmi_decoder_decode(pgmi_ctx* x, const int64_t* ids, int B, const int32_t* slots, const int32_t* positions,
                        void* state, int n_slots, int max_tokens, int n_steps, float* logits, int64_t* next_ids,
                        int64_t* tokens, int use_graph, void* stream) {
    int rc;
    if ((rc = ensure_prepared(x, FAMILY_DECODER))) return rc;
    DecoderState& d = *x->dec;
    if (!ids || !slots || !positions || !logits) return fail(PGMI_E_ARG, "null argument");
    if (n_steps < 1) return fail(PGMI_E_ARG, "n_steps must be >= 1");
    if (n_steps > 1 && !next_ids) return fail(PGMI_E_ARG, "several steps feed their tokens back through next_ids");
    if ((rc = check_state(d, state, n_slots, max_tokens)) || (rc = check_seqs(d, B, slots, n_slots))) return rc;
    for (int b = 0; b < B; ++b)
        if (positions[b] < 0 || (long)positions[b] + n_steps > max_tokens) return fail(PGMI_E_ARG, "state capacity exceeded");
    HIPCHK(hipSetDevice(x->device));
    hipStream_t s = (hipStream_t)stream;
    if ((rc = ensure_workspace(x, B, 1, 1))) return rc;
    size_t need = 0;
    for (const pgmi_layer_spec& l : d.L)
        if (l.mixer == PGMI_MIXER_ATTENTION)
            need = std::max(need, wattn_decode_floats(B, l.heads, r8(l.vdim), wattn_decode_splits(B, l.kv_heads, attn_score(l, {}), max_tokens)));
    if (need > d.part_floats) {
        HIPCHK(hipDeviceSynchronize());
        clear_dgraphs(x);
        if (d.part) (void)hipFree(d.part);
        d.part = nullptr;
        d.part_floats = 0;
        if (hipMalloc(reinterpret_cast<void**>(&d.part), need * 4) != hipSuccess) {
            d.part = nullptr;
            return fail(PGMI_E_NOMEM, "attention partials");
        }
        d.part_floats = need;
    }
    const std::vector<int> ns(slots, slots + B), np(positions, positions + B);
    if (d.known_slot != ns || d.known_pos != np) {
        d.known_slot = ns;  // the copies' sources: alive until overwritten by a later call's own
        d.known_pos = np;
        HIPCHK(hipMemcpyAsync(d.slot, d.known_slot.data(), (size_t)B * 4, hipMemcpyHostToDevice, s));
        HIPCHK(hipMemcpyAsync(d.pos, d.known_pos.data(), (size_t)B * 4, hipMemcpyHostToDevice, s));
    }
    d.known_slot.clear();  // known again once the steps are enqueued
    auto advanced = [&]() {
        d.known_slot = ns;
        d.known_pos = np;
        for (int& p : d.known_pos) p += n_steps;
    };
    int64_t* nx = next_ids ? next_ids : d.d_next;
    auto body = [&](hipStream_t st, const int64_t* first) -> int {
        for (int t = 0; t < n_steps; ++t) {
            const int r = decode_body_rt(x, st, t == 0 ? first : nx, B, state, n_slots, max_tokens, logits, nx,
                                         tokens ? tokens + (long)t * B : nullptr);
            if (r) return r;
        }
        return 0;
    };
    if (!use_graph) {
        if ((rc = body(s, ids))) return rc;
        LAUNCHCHK();
        advanced();
        return 0;
    }
    const int64_t* gids = ids;
    if (ids != next_ids) {  // a stable address for the graph
        HIPCHK(hipMemcpyAsync(d.d_ids, ids, (size_t)B * sizeof(int64_t), hipMemcpyDeviceToDevice, s));
        gids = d.d_ids;
    }
    GraphKey key{B, state, n_slots, max_tokens, logits, next_ids, gids, false, 0, n_steps, tokens};
    GraphEntry& ge = x->graphs[key];
    if (!ge.exec) {
        if (ge.seen++ == 0) {  // first call with this key: run eagerly (sets kernel attributes)
            if ((rc = body(s, gids))) return rc;
            LAUNCHCHK();
            advanced();
            return 0;
        }
        HIPCHK(hipStreamSynchronize(s));
        hipGraph_t g;
        HIPCHK(hipStreamBeginCapture(x->cap_stream, hipStreamCaptureModeThreadLocal));
        rc = body(x->cap_stream, gids);
        HIPCHK(hipStreamEndCapture(x->cap_stream, &g));
        if (rc) {
            (void)hipGraphDestroy(g);
            return rc;
        }
        HIPCHK(hipGraphInstantiate(&ge.exec, g, nullptr, nullptr, 0));
        (void)hipGraphDestroy(g);
    }
    HIPCHK(hipGraphLaunch(ge.exec, s));
    LAUNCHCHK();
    advanced();
    return 0;
}

int pgmi_op_matmul(pgmi_ctx* x, const void* A, int lda, const void* W, int ldw, int M, int N, int K, int act, int mode,
                   const void* bias, void* out, int ldo, int64_t out_bytes, void* scratch, int* split, void* stream) {
    if (!x || !A || !W || !out) return fail(PGMI_E_ARG, "null argument");
    if (M < 1 || N < 1 || K < 8 || K % 8 != 0 || lda < K || ldw < K || lda % 8 != 0 || ldw % 8 != 0)
        return fail(PGMI_E_ARG, "K, lda, ldw must be multiples of 8 with lda, ldw >= K");
    if (act != PGMI_DTYPE_BF16 && act != PGMI_DTYPE_F32) return fail(PGMI_E_ARG, "activations are bf16 or fp32");
    if (mode < 0 || mode > 3) return fail(PGMI_E_ARG, "unknown mode");
    if ((mode == RT_ACT || mode == RT_SWIGLU) && ldo < N) return fail(PGMI_E_ARG, "ldo < N");
    if (mode == RT_SWIGLU && act == PGMI_DTYPE_F32 && !scratch) return fail(PGMI_E_ARG, "fp32 gate|up needs scratch");
    const int sp = matmul_rt((hipStream_t)stream, act == PGMI_DTYPE_F32 ? ACT_F32 : ACT_BF16, A, lda,
                             reinterpret_cast<const uint16_t*>(W), ldw, M, N, K, (RtOut)mode,
                             reinterpret_cast<const uint16_t*>(bias), out, ldo, (size_t)std::max<int64_t>(out_bytes, 0),
                             reinterpret_cast<float*>(scratch));
    if (split) *split = sp;
    LAUNCHCHK();
    return 0;
}

}  // extern "C"
