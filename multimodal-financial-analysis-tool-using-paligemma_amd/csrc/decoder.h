// decoder.h -- host-side launchers of the layered-decoder mechanisms (internal, not the C ABI).
//
// Every launcher takes its sizes and constants as arguments; activations are bf16 (raw uint16_t) or fp32
// (the Act tag), weights are bf16, and residual streams, recurrent states, norms, scores and everything
// inside a recurrence are fp32 in both.  Rows are the step's tokens, sequence after sequence, unpadded.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace pgmi {

enum Act : int { ACT_BF16 = 0, ACT_F32 = 2 };  // PGMI_DTYPE_*

// one sequence of a step: rows [off, off + len) are its positions [start, start + len); slot: its state
struct SeqInfo {
    int off, len, start, slot;
};
// a run of rows of one sequence that one workgroup walks in order; rel: its first row's offset in the
// sequence's rows; nch: chunks of that sequence in this step
struct ChunkInfo {
    int seq, row, len, rel, idx, nch;
};

// ---------------------------------------------------------------- residual streams (hyper-connections)
// X [rows][S][D] fp32.  First X is made (ids: every stream = embed[token] * escale) or updated in place from
// the finished sublayer's output y:  X'[t] = sum_s mix[s][t] X[s] + out[t] y   (y: `ysplit` fp32 slabs, summed).
// (mix == null: X stays as it is.)  Then u = sum_s in[s] X'[s] (in == null: plain sum), split in `groups` equal parts, each over its own root
// mean square, times w -> h.  rows_idx: only these rows (h compact), X left alone.
struct StreamsArgs {
    float* X;
    int rows, S, D;
    const int64_t* ids;
    const uint16_t* E;
    float escale;
    int vocab;
    const float* y;
    int ysplit;
    long ystride;
    const uint16_t* mix;
    const uint16_t* out;
    const uint16_t* in;
    const uint16_t* w;
    int groups;
    float eps;
    void* h;
    int ldh;  // columns D .. ldh-1 are written as zeros
    const int* rows_idx;
    float* tap;  // optional [rows][D]: the summed streams after the update
};
void streams_norm(hipStream_t s, Act act, const StreamsArgs& a);

// ---------------------------------------------------------------- one residual stream
// The outputs of a mixture of experts, folded into the residual row by row: sum_k w[k] (expert sel[k]'s output), where a
// chosen expert >= experts is an identity: its output is the mixture's input h.
struct ExpertMix {
    const void* y;  // [rows * top][ldy] activation type: entry row * top + k
    int ldy;
    const int* sel;  // [rows][top]
    const float* w;  // [rows][top]
    int top, experts;
    const void* h;  // [rows][ldh]
    int ldh;
    const float* gate;  // [rows]: factor of ResidualArgs.y (the shared expert's output), null: 1
};
// X [rows][D] fp32.  First X is made (ids: embed[token] * escale, plus a row of a table indexed by token pairs) or
// updated in place, X += mult (y + mix) with y in `ysplit` fp32 slabs; then h = X over its root mean square times w.
// rows_idx: only these rows (h compact), X left alone.
struct ResidualArgs {
    float* X;
    int rows, D;
    const int64_t* ids;
    const uint16_t* E;
    float escale;
    int vocab;
    // pairs: row (previous * mul_prev + current * mul_cur) mod buckets of `pairs`, row `buckets` at position 0;
    // history [slot][max_tokens] holds every sequence's tokens by position (null: no pairs)
    const uint16_t* pairs;
    int64_t mul_prev, mul_cur;
    int buckets;
    int* history;
    int max_tokens;
    const float* y;  // null: nothing to add from here
    int ysplit;
    long ystride;
    ExpertMix mix;  // mix.y null: none
    float mult;
    const uint16_t* w;  // norm weights [D], or one number
    int w_scalar;
    float eps;
    void* h;  // null: no norm
    int ldh;  // columns D .. ldh-1 are written as zeros
    float* inv;  // optional [rows]: 1 / root mean square (with h null: instead of it)
    const int* rows_idx;
    float* tap;  // optional [rows][D]: X after the update
    int* zero;   // optional: nzero words cleared
    int nzero;
    // where a row stands: packed sequences, or (seqs null) one row per sequence
    const SeqInfo* seqs;
    const int* row_seq;
    const int* slot;
    const int* pos;
    // one row per sequence: h also takes the input convolution's step (taps > 0), see CanonArgs
    const uint16_t* cw;
    int taps;
    float* ring;
};
struct RouteArgs;
void residual_norm(hipStream_t s, Act act, const ResidualArgs& a);
// residual_norm of one row per sequence and bf16 activations with the mixture's router behind it, in one launch:
// logits h . W^T (rows n, then the shared expert's gate), the choice, and the lists (RouteArgs.active given).
bool residual_route_fits(Act act, int rows, int D);
void residual_route(hipStream_t s, const ResidualArgs& a, const uint16_t* W, int ldw, const RouteArgs& r);

// Input convolution over packed rows: n = X * inv * w is what the norm gives, h = n + conv(n),
// conv(n)_t = sum_j cw[:, j] n_(t - taps + 1 + j), zeros before the sequence.  ring [slot][taps][D] fp32 keeps the norm of
// position p in row p % taps; the last taps - 1 of every sequence are written once h is complete.
struct CanonArgs {
    const float* X;
    const float* inv;
    const uint16_t* w;
    int w_scalar;
    int rows, D, taps;
    const uint16_t* cw;  // [D][taps]
    float* ring;
    void* h;
    int ldh;
    const SeqInfo* seqs;
    int nseq;
    const ChunkInfo* chunks;
    int nchunk;
};
void canon(hipStream_t s, Act act, const CanonArgs& a);

// ---------------------------------------------------------------- mixture of experts
// z: fp32 slabs [split][rows][ldz], summed: columns 0 .. n-1 the router's logits, column n the shared expert's gate (gate
// != null).  Scores are their softmax; choice = score + correction picks the groups (largest choice of a group, `keep` of
// `groups` equal ones) and the top experts inside them; weights are the scores.  Lists: list[e * cap ..] the entries
// (row * top + k) of expert e < experts in any order, cnt[e] how many (zero before the launch).
struct RouteArgs {
    const float* z;
    int split;
    long zstride;
    int ldz, rows, n, experts, top, groups, keep;
    const uint16_t* correction;
    int* sel;
    float* w;
    float* gate;
    int* cnt;
    int* list;
    int cap;
    int* active;  // residual_route: active[1 .. active[0]] are the experts used, -1: none (active[0] is zero before)
};
constexpr int kRouteRows = 16;  // most rows of residual_route and experts_skinny
constexpr int kMaxExperts = 512;  // identity experts included: a workgroup's choice scores fit LDS
void route(hipStream_t s, const RouteArgs& a);

// One product of every expert over the rows that chose it: entry -> row entry / gather of A (gather: `top` where A is
// the mixture's input, 1 where it is per entry), W + e * wstride, out row = entry.
enum ExpertMode : int {
    EX_SWIGLU = 0,  // silu(A . W_gate^T) * (A . W_up^T), W = N gate rows, then N up rows
    EX_STORE = 1,
};
struct ExpertArgs {
    const void* A;
    int lda, gather;
    const uint16_t* W;
    int ldw;
    long wstride;
    int N, K;
    void* out;
    int ldo;  // columns N .. ldo-1 are written as zeros
    const int* cnt;
    const int* list;
    int cap, experts, entries;  // entries: rows * top
    // experts_skinny: the used experts (RouteArgs.active); the shared expert rides along, its rows 0 .. B-1 (Wsh null: none)
    const int* active;
    const uint16_t* Wsh;
    int ldwsh, Nsh, Ksh;
    const void* Ash;
    int ldash, B;
    void* outsh;
    int ldosh;
};
void experts_rt(hipStream_t s, Act act, ExpertMode mode, const ExpertArgs& a);
// the same for up to kRouteRows rows of bf16 activations, the shared expert included (EX_STORE: its output is fp32)
void experts_skinny(hipStream_t s, ExpertMode mode, const ExpertArgs& a);

// ---------------------------------------------------------------- matrix products, any M, N, K (K a multiple of 8)
// C = A [M][lda] . W [N][ldw]^T
enum RtOut : int {
    RT_ACT = 0,     // activation type, + bias (bf16 [N], optional), [M][ldo]
    RT_F32 = 1,     // fp32 [M][N] (one slab)
    RT_SLABS = 2,   // fp32 partial slabs [split][M][N]; the split is returned
    RT_SWIGLU = 3,  // activation type, silu(A . W_gate^T) * (A . W_up^T); W = gate rows, then N up rows
};
int matmul_rt(hipStream_t s, Act act, const void* A, int lda, const uint16_t* W, int ldw, int M, int N, int K,
              RtOut mode, const uint16_t* bias, void* out, int ldo, size_t out_bytes, float* scratch);

// ---------------------------------------------------------------- selective scan (Mamba)
// xz rows [x: C | z: C] (activation type); taps state fp32 [slot][K-1][C]
void conv_silu(hipStream_t s, Act act, const void* xz, int ldxz, int C, int K, const uint16_t* w, const uint16_t* b,
               const SeqInfo* seqs, int nseq, const ChunkInfo* chunks, int nchunk, float* taps, void* out,
               int ldo);
// slabs [split][rows][R + 2N] -> dt_low (activation type, ldd, zero-padded) and B|C fp32 [rows][2N]
void scan_inputs(hipStream_t s, Act act, const float* slabs, int split, int rows, int R, int N, void* dtl, int ldd,
                 float* bc);
struct ScanArgs {
    const float* dt;      // [rows][C]: W_dt dt (before bias and softplus)
    const uint16_t* dtb;  // [C]
    const void* x;        // [rows][ldx], after the convolution
    int ldx;
    const void* z;        // [rows][ldz]
    int ldz;
    const float* bc;      // [rows][2N]
    const uint16_t* A_log;  // [C][N]
    const uint16_t* Dw;     // [C]
    float* state;           // [slot][C][N]
    float* cstate;          // [chunk][C][N] scratch
    float* csum;            // [chunk][C] scratch
    void* y;                // [rows][ldy]
    int ldy;
    int C, N;
    const SeqInfo* seqs;
    int nseq;
    const ChunkInfo* chunks;
    int nchunk;
    bool multi;  // some sequence has more than one chunk
};
int scan_max_state();
void selective_scan(hipStream_t s, Act act, const ScanArgs& a);

// ---------------------------------------------------------------- minimal gated recurrence (minGRU)
// zug rows [z: C | u: C | g: C]; state fp32 [slot][C]; y = S_t silu(g)
struct GruArgs {
    const void* zug;
    int ld;
    float* state;
    float* cstate;  // [chunk][2][C] scratch
    void* y;
    int ldy;
    int C;
    const SeqInfo* seqs;
    int nseq;
    const ChunkInfo* chunks;
    int nchunk;
    bool multi;
};
void mingru_scan(hipStream_t s, Act act, const GruArgs& a);

// ---------------------------------------------------------------- windowed attention
// qkv rows [q: H d | k: G d | v: G e] (no k and v when own_kv is false: the cache is another layer's).  What the cache
// holds: K [slot][G][max_tokens][dp] after head norm and rotation, V [slot][G][max_tokens][ep] after head norm,
// activation type, dp / ep = d / e rounded up to 8 with zero pads.
struct WAttnHeads {
    int H, G, d, e, dp, ep;
    bool own_kv;
    bool qk_norm, v_norm;  // heads over their root mean square
    float eps;
    const double* turns;   // [rot / 2] turns per position of the pairs (2i, 2i + 1) of q and k
    int rot;               // rotated leading dims, 0: none
};
// Which keys a query sees, and what becomes of its score q . k scale:
//   position i sees j <= i with i - j < window or j < keep
//   cap > 0: cap tanh(score / cap);  r1: r1[h] ln(1 + r2[h] (i - j)) is taken off (one of the two at most)
struct WAttnScore {
    int window, keep;
    float scale, cap;
    const uint16_t* r1;  // [H], null: no distance bias
    const uint16_t* r2;
};
struct WAttnArgs {
    WAttnHeads hd;
    WAttnScore sc;
    const void* qkv;
    int ldqkv;
    void* q;  // queries after norm and rotation [rows][H][dp]
    void* kc;
    void* vc;
    int max_tokens;
    void* o;  // [rows][ldo], head-major H * e
    int ldo;
    int rows;
    const SeqInfo* seqs;
    int nseq;
    const int* row_seq;  // [rows]
    const ChunkInfo* tiles;
    int ntile;
};
void wattn_append(hipStream_t s, Act act, const WAttnArgs& a);
constexpr int kWAttnRows = 64;  // (position, query head of the group) pairs per prefill tile: ChunkInfo.rel of `tiles`
void wattn_prefill(hipStream_t s, Act act, const WAttnArgs& a);

// one new token per sequence: row b of qkv (activation type [B][ldqkv], biases added) is position pos[b] of slot[b]; appends
// its k and v, attends, and leaves the heads' outputs in o [B][ldo].  part: fp32 scratch of wattn_decode_floats().
struct WAttnDecodeArgs {
    WAttnHeads hd;
    WAttnScore sc;
    const void* qkv;
    int ldqkv;
    void* kc;
    void* vc;
    int max_tokens;
    void* o;
    int ldo;
    int B;
    const int* slot;
    const int* pos;
    float* part;
    int nsplit;
};
int wattn_decode_splits(int B, int G, const WAttnScore& sc, int max_tokens);
size_t wattn_decode_floats(int B, int H, int ep, int nsplit);
void wattn_decode(hipStream_t s, Act act, const WAttnDecodeArgs& a);

// ---------------------------------------------------------------- one token per sequence: fused projections
// y = W x for a few rows, one launch per projection, the epilogue being the step that follows the projection.
enum GemvRtForm : int {
    GF_NONE = 0,    // too many rows: matmul_rt and the step kernels below
    GF_STREAM = 1,  // weight-streaming GEMV; the input may be the streams' next read and norm (as streams_norm)
    GF_SKINNY = 2,  // MFMA, up to gemv_rt_max_batch() rows of bf16 activations
};
enum GemvRtMode : int {
    GR_ACT = 0,      // out (activation type) = acc + bias
    GR_CONV = 1,     // rows < C: convolution step with the taps in place, silu -> out; rows >= C -> out2
    GR_GRU = 2,      // N channels, rows c, N + c, 2N + c (z, u, g): one minGRU step, state in place -> out
    GR_SWIGLU = 3,   // N channels, rows n, N + n: silu(gate) * up -> out
    GR_STREAMS = 4,  // X'[t] = sum_s mix[s][t] X[s] + wout[t] acc, in place
    GR_LOGITS = 5,   // fp32 out + (GF_STREAM) per-workgroup argmax partials
    GR_F32 = 6,      // fp32 out; GF_SKINNY: `split` partial slabs [split][B][ldo]
};
struct GemvRtArgs {
    GemvRtForm form;
    int B, N, K;  // N: outputs (rows of W, or channels); K: padded to 8
    const uint16_t* W;
    int ldw;
    const void* x;  // [B][ldx] activations, or null: the streams' read
    int ldx;
    float* X;  // [B][S][D]
    int S, D, groups;
    float eps;
    const uint16_t* in;
    const uint16_t* nw;
    const uint16_t* bias;
    void* out;
    int ldo;
    void* out2;
    int ldo2;
    // GR_CONV
    int C, taps_k;
    const uint16_t* cw;
    const uint16_t* cb;
    // GR_CONV taps [slot][taps_k - 1][C], GR_GRU state [slot][N]
    float* state;
    const int* slot;
    const int* pos;
    // GR_STREAMS; mix null: one stream, X += mult acc
    const uint16_t* mix;
    const uint16_t* wout;
    float mult;
    int split;  // GR_F32
    // GR_LOGITS
    float* pmax;
    int* pidx;
};
int gemv_rt_max_batch();
int gemv_rt_parts();  // words of pmax / pidx
GemvRtForm gemv_rt_form(int B, Act act, int streams, int width);
bool gemv_rt_fits(GemvRtForm form, int K, Act act);
int gemv_rt_split(GemvRtForm form, int N, int K);  // slabs of a GR_F32 product
int gemv_rt_blocks(const GemvRtArgs& a, GemvRtMode mode);
void gemv_rt(hipStream_t s, Act act, GemvRtMode mode, const GemvRtArgs& a);

// one token of the convolution for B rows of xz (as conv_silu, taps in place)
void conv_step(hipStream_t s, Act act, const void* xz, int ldxz, int B, int C, int K, const uint16_t* w,
               const uint16_t* b, float* taps, const int* slot, const int* pos, void* out, int ldo);
// one token of the selective scan for B rows: slabs [split][B][R + 2N] hold dt_low | B | C, dt = softplus(Wdt dt_low
// + dtb) is formed here; y = (S C + D x) silu(z)
struct ScanStepArgs {
    const float* slabs;
    int split;
    const uint16_t* Wdt;
    int ldwdt;
    const uint16_t* dtb;
    const void* x;
    int ldx;
    const void* z;
    int ldz;
    const uint16_t* A_log;
    const uint16_t* Dw;
    float* state;
    const int* slot;
    const int* pos;
    void* y;
    int ldy;
    int B, C, N, R;
};
void scan_step(hipStream_t s, Act act, const ScanStepArgs& a);

// one token of the gated recurrence for B rows of zug (as mingru_scan)
void gru_step(hipStream_t s, Act act, const void* zug, int ld, int B, int C, float* state, const int* slot,
              const int* pos, void* y, int ldy);

// the end of a decode step: next[b] from the argmax partials (nparts > 0) or as already written (0), also to
// hist when given; every sequence's position advances by one
void decode_finish(hipStream_t s, int B, const float* pmax, const int* pidx, int nparts, int64_t* next, int64_t* hist,
                   int* pos);
}  // namespace pgmi
