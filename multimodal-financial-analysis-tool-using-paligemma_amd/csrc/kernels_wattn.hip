// kernels_wattn.hip -- grouped-query attention over a sliding window and, optionally, the sequence's first tokens; a
// logarithmic distance bias or a tanh cap on the scores; heads over their root mean squares; rotary positions; any head
// sizes.  Scores, weights, norms, positions and angles are fp32 (angles reduced in fp64).
//
//   k_append    norms and rotates the heads of a prefill's rows, writes the key / value rows into the cache
//   k_wattn     plain form, any size and both activation types: one workgroup per (row, head), online softmax
//   k_wattn_m   bf16 MFMA form: 64 (position, head) pairs per workgroup against 64-key tiles of one key/value head
//   k_wattn_d   one new token per sequence: keys split over workgroups, partials merged by k_wattn_dc
//   k_wattn_dm  the same on bf16 MFMA
#include <algorithm>

#include "act.h"
#include "decoder.h"

namespace pgmi {

namespace {

typedef short s4v __attribute__((ext_vector_type(4)));
constexpr float kLog2e = 1.4426950408889634f;
constexpr float kNone = -1e30f;  // running maximum before any key: finite, so exp2(-inf - kNone) is 0

// score modes
constexpr int SC_PLAIN = 0;  // scale, and a cap where sc.cap > 0
constexpr int SC_BIAS = 1;   // scale and distance bias
constexpr int SC_CAPPED = 2; // a cap so small that exp(+-cap) and sums of it fit fp32: no running maximum
constexpr float kCapFixed = 66.0f;  // nats: 2^95 times 2^20 keys times values in fp32

// score in powers of two: dot * c1 - r1 log2(1 + r2 dist)
__device__ __forceinline__ float biased(float dot, float c1, float r1, float r2, float dist) {
    return dot * c1 - r1 * __builtin_amdgcn_logf(fmaf(r2, dist, 1.0f));
}
// cap log2(e) tanh(x) from exp(2x): cap2 = cap log2(e), d2 = dot * 2 log2(e) scale / cap
__device__ __forceinline__ float capped(float d2, float cap2) {
    return fmaf(-2.0f * cap2, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(d2)), cap2);
}
// a head's score constants; fast() on the hardware's transcendentals, exact() on the library's
template <int SC>
struct Score {
    float c1, cap2, r1, r2;
    __device__ __forceinline__ Score(const WAttnScore& s, int h) {
        cap2 = s.cap * kLog2e;
        c1 = (SC == SC_CAPPED || (SC == SC_PLAIN && s.cap > 0.0f)) ? 2.0f * kLog2e * s.scale / s.cap : s.scale * kLog2e;
        r1 = SC == SC_BIAS ? bf2f(s.r1[h]) : 0.0f;
        r2 = SC == SC_BIAS ? bf2f(s.r2[h]) : 0.0f;
    }
    __device__ __forceinline__ float fast(float dot, float dist) const {
        if constexpr (SC == SC_BIAS) return biased(dot, c1, r1, r2, dist);
        else if constexpr (SC == SC_CAPPED) return capped(dot * c1, cap2);
        else return cap2 > 0.0f ? capped(dot * c1, cap2) : dot * c1;
    }
    __device__ __forceinline__ float exact(float dot, float dist) const {
        if constexpr (SC == SC_BIAS) return dot * c1 - r1 * (log1pf(r2 * dist) * kLog2e);
        else return cap2 > 0.0f ? cap2 * tanhf(dot * c1 * (0.5f / kLog2e)) : dot * c1;
    }
};

// n-th key a query at i sees, in order: the kept first tokens before the window, then the window
struct Keys {
    int kept, lo, n;
    __device__ __forceinline__ Keys(const WAttnScore& s, int i) {
        lo = max(0, i - s.window + 1);
        kept = min(s.keep, lo);
        n = kept + i - lo + 1;
    }
    __device__ __forceinline__ int at(int v) const { return v < kept ? v : v - kept + lo; }
};

// pair p of a head at position pos: (u, v) turned
__device__ __forceinline__ void rotate(const double* turns, int p, int pos, float& u, float& v) {
    double t = turns[p] * (double)pos;
    t -= rint(t);
    float s, c;
    sincospif(2.0f * (float)t, &s, &c);
    const float x = u;
    u = x * c - v * s;
    v = v * c + x * s;
}

// ---------------------------------------------------------------- append
// LPH lanes per head of a row (8 elements each when V == 8: head sizes that are multiples of 8)
template <typename T, int LPH, int V>
__global__ void __launch_bounds__(256) k_append(WAttnArgs a) {
    const WAttnHeads& w = a.hd;
    const int row = blockIdx.x, sub = threadIdx.x % LPH;
    const int head = blockIdx.y * (256 / LPH) + threadIdx.x / LPH, NH = w.own_kv ? w.H + 2 * w.G : w.H;
    const SeqInfo q = a.seqs[a.row_seq[row]];
    const int pos = q.start + (row - q.off);
    const T* src = reinterpret_cast<const T*>(a.qkv) + (long)row * a.ldqkv;
    const int hd = head < NH ? head : NH - 1;
    T* dst;
    int n, np, rot = w.rot;
    bool norm = w.qk_norm;
    if (hd < w.H) {
        src += hd * w.d; n = w.d; np = w.dp;
        dst = reinterpret_cast<T*>(a.q) + ((long)row * w.H + hd) * w.dp;
    } else if (hd < w.H + w.G) {
        const int g = hd - w.H;
        src += w.H * w.d + g * w.d; n = w.d; np = w.dp;
        dst = reinterpret_cast<T*>(a.kc) + (((long)q.slot * w.G + g) * a.max_tokens + pos) * w.dp;
    } else {
        const int g = hd - w.H - w.G;
        src += (w.H + w.G) * w.d + g * w.e; n = w.e; np = w.ep;
        dst = reinterpret_cast<T*>(a.vc) + (((long)q.slot * w.G + g) * a.max_tokens + pos) * w.ep;
        norm = w.v_norm;
        rot = 0;
    }
    float ss = 0.0f;
    for (int i = sub * V; i < n; i += LPH * V) {
        if constexpr (V == 8) {
            float v[8];
            ld8(src + i, v);
#pragma unroll
            for (int t = 0; t < 8; ++t) ss = fmaf(v[t], v[t], ss);
        } else {
            const float v = ldf(src + i);
            ss = fmaf(v, v, ss);
        }
    }
#pragma unroll
    for (int o = 1; o < LPH; o <<= 1) ss += __shfl_xor(ss, o, 64);
    const float inv = norm ? 1.0f / sqrtf(ss / (float)n + w.eps) : 1.0f;
    if (head >= NH) return;
    for (int i = sub * V; i < np; i += LPH * V) {
        if constexpr (V == 8) {
            float v[8];
            ld8(src + i, v);
#pragma unroll
            for (int t = 0; t < 8; ++t) v[t] *= inv;
#pragma unroll
            for (int t = 0; t < 8; t += 2)
                if (i + t < rot) rotate(w.turns, (i + t) / 2, pos, v[t], v[t + 1]);
            st8(dst + i, v);
        } else {
            float u = i < n ? ldf(src + i) * inv : 0.0f;
            if (i < rot) {
                float o = ldf(src + (i ^ 1)) * inv;
                if (i & 1) { rotate(w.turns, i / 2, pos, o, u); }
                else { rotate(w.turns, i / 2, pos, u, o); }
            }
            stf(dst + i, u);
        }
    }
}

template <typename T>
void append_t(hipStream_t s, const WAttnArgs& a) {
    const int NH = a.hd.own_kv ? a.hd.H + 2 * a.hd.G : a.hd.H;
    if (a.hd.d % 8 == 0 && a.hd.e % 8 == 0)
        hipLaunchKernelGGL((k_append<T, 16, 8>), dim3(a.rows, (NH + 15) / 16), dim3(256), 0, s, a);
    else
        hipLaunchKernelGGL((k_append<T, 64, 1>), dim3(a.rows, (NH + 3) / 4), dim3(256), 0, s, a);
}

// ---------------------------------------------------------------- plain form
template <typename T, int SC>
__global__ void __launch_bounds__(256) k_wattn(WAttnArgs a) {
    extern __shared__ float sm[];
    const WAttnHeads& w = a.hd;
    float* qs = sm;              // [dp]
    float* p = qs + w.dp;        // [256]
    float* red = p + 256;        // [8]
    const int row = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const SeqInfo q = a.seqs[a.row_seq[row]];
    const int i = q.start + (row - q.off), g = h / (w.H / w.G);
    const T* qp = reinterpret_cast<const T*>(a.q) + ((long)row * w.H + h) * w.dp;
    for (int k = tid; k < w.dp; k += 256) qs[k] = ldf(qp + k);
    __syncthreads();
    const T* kc = reinterpret_cast<const T*>(a.kc) + ((long)q.slot * w.G + g) * a.max_tokens * w.dp;
    const T* vc = reinterpret_cast<const T*>(a.vc) + ((long)q.slot * w.G + g) * a.max_tokens * w.ep;
    const Score<SC> score(a.sc, h);
    const Keys keys(a.sc, i);
    float m = kNone, l = 0.0f;
    constexpr int EM = 8;  // value columns per thread: e <= 2048
    float acc[EM] = {};
    for (int j0 = 0; j0 < keys.n; j0 += 256) {
        float s = -INFINITY;
        if (j0 + tid < keys.n) {
            const int j = keys.at(j0 + tid);
            const T* kr = kc + (long)j * w.dp;
            float dot = 0.0f;
            for (int k = 0; k < w.d; ++k) dot = fmaf(qs[k], ldf(kr + k), dot);
            s = score.exact(dot, (float)(i - j));
        }
        float t = wave_max(s);
        if (lane == 0) red[wave] = t;
        __syncthreads();
        t = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
        const float mn = fmaxf(m, t), alpha = exp2f(m - mn);
        const float e = exp2f(s - mn);
        p[tid] = e;
        const float ws = wave_sum(e);
        if (lane == 0) red[4 + wave] = ws;
        __syncthreads();
        l = l * alpha + red[4] + red[5] + red[6] + red[7];
        m = mn;
        const int n = min(256, keys.n - j0);
#pragma unroll
        for (int v = 0; v < EM; ++v) {
            const int col = tid + 256 * v;
            if (col < w.e) {
                float o = acc[v] * alpha;
                for (int k = 0; k < n; ++k) o = fmaf(p[k], ldf(vc + (long)keys.at(j0 + k) * w.ep + col), o);
                acc[v] = o;
            }
        }
        __syncthreads();
    }
    T* o = reinterpret_cast<T*>(a.o) + (long)row * a.ldo;
#pragma unroll
    for (int v = 0; v < EM; ++v) {
        const int col = tid + 256 * v;
        if (col < w.e) stf(o + h * w.e + col, acc[v] / l);
    }
    if (h == w.H - 1)
        for (int k = w.H * w.e + tid; k < a.ldo; k += 256) stf(o + k, 0.0f);
}

// ---------------------------------------------------------------- bf16 MFMA form
// Scores are computed transposed, S^T = K Q^T, so that a lane holds one query row (column lane & 15) and, after
// two 16-key tiles, exactly the 8 weights its B fragment of O^T = V^T P^T needs (the contraction order is free:
// slot 8g + i is key 4g + i of the first tile for i < 4, of the second for i >= 4).  V^T fragments are
// transposed LDS reads of the row-major V tile.
template <int DQ, int DV, int SC>
__global__ void __launch_bounds__(256) k_wattn_m(WAttnArgs a) {
    const WAttnHeads& w = a.hd;
    constexpr int KT = 64;                 // keys per tile
    constexpr int KS = DQ + 8, VS = DV + 8;  // LDS row strides (elements)
    constexpr int KQ = KT * DQ / 8 / 256, VQ = KT * DV / 8 / 256;  // 16-byte pieces per thread
    __shared__ __attribute__((aligned(16))) uint16_t Ks[KT * KS];
    __shared__ __attribute__((aligned(16))) uint16_t Vs[KT * VS];
    const ChunkInfo tl = a.tiles[blockIdx.x];
    const SeqInfo sq = a.seqs[tl.seq];
    const int g = blockIdx.y, R = w.H / w.G;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane & 15, lg = lane >> 4;
    const int nrow = sq.len * R;
    // this lane's query row
    const int fr = tl.rel + wave * 16 + li;
    const bool ok = fr < nrow;
    const int frc = ok ? fr : nrow - 1;
    const int prow = frc / R, hh = frc % R, h = g * R + hh;
    const int i = sq.start + prow;
    const uint16_t* qp = reinterpret_cast<const uint16_t*>(a.q) + ((long)(sq.off + prow) * w.H + h) * w.dp;
    short8 qf[DQ / 32];
#pragma unroll
    for (int c = 0; c < DQ / 32; ++c) {
        const int k = c * 32 + 8 * lg;
        const uint4 v = ldg16_sel(qp + k, k < w.dp, qp);
        qf[c] = __builtin_bit_cast(short8, v);
    }
    const Score<SC> score(a.sc, h);
    const float r1 = score.r1, r2 = score.r2, c1 = score.c1;
    const int window = a.sc.window, keep = a.sc.keep;
    // keys the tile's rows see: [lo, hi], and the kept ones before them: [0, kept)
    const int last = min(tl.rel + kWAttnRows, nrow) - 1;
    const int lo = max(0, sq.start + tl.rel / R - window + 1), hi = sq.start + last / R;
    const int kept = min(keep, lo);
    // positions of this wave's first and last rows
    const int wfirst = sq.start + min(tl.rel + wave * 16, nrow - 1) / R;
    const int wlast = sq.start + min(tl.rel + wave * 16 + 15, nrow - 1) / R;
    const uint16_t* kc = reinterpret_cast<const uint16_t*>(a.kc) + ((long)sq.slot * w.G + g) * a.max_tokens * w.dp;
    const uint16_t* vc = reinterpret_cast<const uint16_t*>(a.vc) + ((long)sq.slot * w.G + g) * a.max_tokens * w.ep;
    f32x4 o[DV / 16];
#pragma unroll
    for (int c = 0; c < DV / 16; ++c) o[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = SC == SC_CAPPED ? 0.0f : kNone, l = 0.0f;
    uint4 kr[KQ], vr[VQ];
    auto gload = [&](int j0) {
#pragma unroll
        for (int x = 0; x < KQ; ++x) {
            const int e = tid + 256 * x, r = e / (DQ / 8), k = (e % (DQ / 8)) * 8;
            const int j = min(j0 + r, hi);
            kr[x] = ldg16_sel(kc + (long)j * w.dp + k, k < w.dp, kc);
        }
#pragma unroll
        for (int x = 0; x < VQ; ++x) {
            const int e = tid + 256 * x, r = e / (DV / 8), k = (e % (DV / 8)) * 8;
            const int j = min(j0 + r, hi);
            vr[x] = ldg16_sel(vc + (long)j * w.ep + k, k < w.ep, vc);
        }
    };
    auto next = [&](int j0) { return j0 < kept && j0 + KT >= kept ? lo : j0 + KT; };  // kept keys end before lo
    const int first = kept > 0 ? 0 : lo;
    gload(first);
    for (int j0 = first, jn; j0 <= hi; j0 = jn) {
        jn = next(j0);
        __syncthreads();  // the previous tile's reads are done
#pragma unroll
        for (int x = 0; x < KQ; ++x) {
            const int e = tid + 256 * x, r = e / (DQ / 8), k = (e % (DQ / 8)) * 8;
            *reinterpret_cast<uint4*>(Ks + r * KS + k) = kr[x];
        }
#pragma unroll
        for (int x = 0; x < VQ; ++x) {
            const int e = tid + 256 * x, r = e / (DV / 8), k = (e % (DV / 8)) * 8;
            *reinterpret_cast<uint4*>(Vs + r * VS + k) = vr[x];
        }
        __syncthreads();
        if (jn <= hi) gload(jn);
        if (j0 > wlast || (j0 + KT <= wfirst - window + 1 && j0 >= keep)) continue;  // no row of this wave sees the tile
        f32x4 st[4];
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            st[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c) {
                const short8 kf = *reinterpret_cast<const short8*>(Ks + (t * 16 + li) * KS + c * 32 + 8 * lg);
                st[t] = mfma16(kf, qf[c], st[t]);
            }
        }
        const bool head = j0 < kept;  // kept keys: every row sees those before lo
        float mt = m;
        // 1 + r2 (i - j) for key j0 + 4 lg, less r2 per key after it
        const float x0 = fmaf(r2, (float)(i - j0 - 4 * lg), 1.0f);
        auto value = [&](float dot, int k) {
            if constexpr (SC == SC_BIAS) return fmaf(-r1, __builtin_amdgcn_logf(fmaf(-r2, (float)k, x0)), dot * c1);
            else return score.fast(dot, 0.0f);
        };
        if (head ? j0 + KT <= kept : j0 + KT - 1 <= wfirst && (wlast - j0 < window || j0 + KT <= keep)) {  // no mask
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) st[t][r] = value(st[t][r], t * 16 + r);
        } else {
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int j = j0 + t * 16 + 4 * lg + r, dist = i - j;
                    const bool see = head ? j < kept : dist >= 0 && (dist < window || j < keep);
                    const float s = value(st[t][r], t * 16 + r);
                    st[t][r] = see ? s : -INFINITY;
                }
        }
        float alpha = 1.0f;
        if constexpr (SC != SC_CAPPED) {
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) mt = fmaxf(mt, st[t][r]);
            mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
            mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
            alpha = __builtin_amdgcn_exp2f(m - mt);
            m = mt;
        }
        float ls = 0.0f;
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                st[t][r] = __builtin_amdgcn_exp2f(SC == SC_CAPPED ? st[t][r] : st[t][r] - m);
                ls += st[t][r];
            }
        l = l * alpha + ls;  // this lane's keys; summed over the lane groups at the end
        if (SC != SC_CAPPED && __any(alpha != 1.0f)) {
#pragma unroll
            for (int c = 0; c < DV / 16; ++c)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[c][r] *= alpha;
        }
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            short8 pf;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                pf[r] = (short)f2bf(st[2 * u][r]);
                pf[4 + r] = (short)f2bf(st[2 * u + 1][r]);
            }
#pragma unroll
            for (int c = 0; c < DV / 16; ++c) {
                uint16_t* vp = Vs + (u * 32 + 4 * lg + (li >> 2)) * VS + c * 16 + 4 * (li & 3);
                const s4v lo4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(vp));
                const s4v hi4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(vp + 16 * VS));
                const short8 vf = {lo4[0], lo4[1], lo4[2], lo4[3], hi4[0], hi4[1], hi4[2], hi4[3]};
                o[c] = mfma16(vf, pf, o[c]);
            }
        }
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (!ok) return;
    const float inv = 1.0f / l;
    uint16_t* op = reinterpret_cast<uint16_t*>(a.o) + (long)(sq.off + prow) * a.ldo + h * w.e;
#pragma unroll
    for (int c = 0; c < DV / 16; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int col = c * 16 + 4 * lg + r;
            if (col < w.e) op[col] = f2bf(o[c][r] * inv);
        }
    if (h == w.H - 1 && lg == 0)
        for (int k = w.H * w.e; k < a.ldo; ++k) reinterpret_cast<uint16_t*>(a.o)[(long)(sq.off + prow) * a.ldo + k] = 0;
}

// the score mode of a layer on the hardware's transcendentals
int score_mode(const WAttnScore& sc) { return sc.r1 ? SC_BIAS : sc.cap > 0.0f && sc.cap <= kCapFixed ? SC_CAPPED : SC_PLAIN; }

template <int DQ, int DV>
void run_m(hipStream_t s, const WAttnArgs& a) {
    const dim3 grid(a.ntile, a.hd.G);
    const int mode = score_mode(a.sc);
    if (mode == SC_BIAS) hipLaunchKernelGGL((k_wattn_m<DQ, DV, SC_BIAS>), grid, dim3(256), 0, s, a);
    else if (mode == SC_CAPPED) hipLaunchKernelGGL((k_wattn_m<DQ, DV, SC_CAPPED>), grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((k_wattn_m<DQ, DV, SC_PLAIN>), grid, dim3(256), 0, s, a);
}
template <int DQ>
void run_mv(hipStream_t s, const WAttnArgs& a) {
    if (a.hd.ep <= 64) run_m<DQ, 64>(s, a);
    else if (a.hd.ep <= 96) run_m<DQ, 96>(s, a);
    else if (a.hd.ep <= 128) run_m<DQ, 128>(s, a);
    else run_m<DQ, 256>(s, a);
}

// ---------------------------------------------------------------- one token per sequence
constexpr int DK = 64;  // keys per tile

// grid (split, G, B).  RB: query heads of the group handled at once (registers).
// part record of (b, head, split): [ep] weighted values, then running maximum, then sum of weights
template <typename T, int RB, int SC>
__global__ void __launch_bounds__(256) k_wattn_d(WAttnDecodeArgs a) {
    extern __shared__ float sm[];
    const WAttnHeads& w = a.hd;
    const int R = w.H / w.G;
    float* qs = sm;                 // [R][dp] normalised queries
    float* ps = qs + R * w.dp;      // [RB][DK] scores, then weights
    float* st = ps + RB * DK;       // [RB][4]: running max, sum, alpha
    float* red = st + RB * 4;       // [256][8] cross-group reduction
    const int g = blockIdx.y, b = blockIdx.z, sp = blockIdx.x;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int slot = a.slot[b], i = a.pos[b];
    const Keys keys(a.sc, i);  // k0, k1, j below count the keys this query sees
    const int per = ((keys.n + a.nsplit - 1) / a.nsplit + DK - 1) / DK * DK;
    const int k0 = sp * per, k1 = min(keys.n, k0 + per);  // empty when k0 >= k1
    const T* qkv = reinterpret_cast<const T*>(a.qkv) + (long)b * a.ldqkv;
    const int rs = w.ep + 2;
    float* part = a.part + (((long)b * w.H + g * R) * a.nsplit + sp) * rs;
    if (k0 >= k1) {
        for (int r = tid; r < R; r += 256) {
            part[(long)r * a.nsplit * rs + w.ep] = kNone;
            part[(long)r * a.nsplit * rs + w.ep + 1] = 0.0f;
        }
        return;
    }
    T* kc = reinterpret_cast<T*>(a.kc) + ((long)slot * w.G + g) * a.max_tokens * w.dp;
    T* vc = reinterpret_cast<T*>(a.vc) + ((long)slot * w.G + g) * a.max_tokens * w.ep;
    // n elements of a head row by one wave, normed and rotated, rounded to T as the prefill form rounds them: put(k, v)
    auto head_row = [&](const T* src, int n, int np, bool norm, int rot, auto put) {
        float ss = 0.0f;
        for (int k = lane; k < n; k += 64) ss = fmaf(ldf(src + k), ldf(src + k), ss);
        const float inv = norm ? 1.0f / sqrtf(wave_sum(ss) / (float)n + w.eps) : 1.0f;
        for (int k = 2 * lane; k < np; k += 128) {  // np is even
            float u = k < n ? ldf(src + k) * inv : 0.0f, v = k + 1 < n ? ldf(src + k + 1) * inv : 0.0f;
            if (k < rot) rotate(w.turns, k / 2, i, u, v);
            put(k, u);
            put(k + 1, v);
        }
    };
    for (int r = wave; r < R; r += 4)
        head_row(qkv + (g * R + r) * w.d, w.d, w.dp, w.qk_norm, w.rot, [&](int k, float v) {
            T t;
            stf(&t, v);
            qs[r * w.dp + k] = ldf(&t);
        });
    if (k1 == keys.n && w.own_kv) {  // this workgroup's keys include the new one: write its cache rows
        if (wave == 0)
            head_row(qkv + w.H * w.d + g * w.d, w.d, w.dp, w.qk_norm, w.rot,
                     [&](int k, float v) { stf(kc + (long)i * w.dp + k, v); });
        else if (wave == 1)
            head_row(qkv + (w.H + w.G) * w.d + g * w.e, w.e, w.ep, w.v_norm, 0,
                     [&](int k, float v) { stf(vc + (long)i * w.ep + k, v); });
        __threadfence_block();
    }
    __syncthreads();
    // scores: LPK lanes share a key, 8 elements each per step
    int LPK = 1;
    while (LPK < 64 && LPK * 8 < w.dp) LPK <<= 1;
    const int kl = lane % LPK, kw = wave * (64 / LPK) + lane / LPK, kstep = 4 * (64 / LPK);
    // weighted values: CPV threads span the columns (8 each), the rest split the keys
    const int nch = w.ep / 8;
    int CPV = 1;
    while (CPV < 256 && CPV < nch) CPV <<= 1;
    const int vch = tid % CPV, vk = tid / CPV, vkn = 256 / CPV;
    for (int r0 = 0; r0 < R; r0 += RB) {
        const int nr = min(RB, R - r0);
        float acc[RB][8];
#pragma unroll
        for (int r = 0; r < RB; ++r)
#pragma unroll
            for (int v = 0; v < 8; ++v) acc[r][v] = 0.0f;
        if (tid < RB) { st[tid * 4] = kNone; st[tid * 4 + 1] = 0.0f; }
        __syncthreads();
        for (int j0 = k0; j0 < k1; j0 += DK) {
            for (int kk = kw; kk < DK; kk += kstep) {
                const int j = j0 + kk;
                float dot[RB];
#pragma unroll
                for (int r = 0; r < RB; ++r) dot[r] = 0.0f;
                if (j < k1)
                    for (int c = kl * 8; c < w.dp; c += LPK * 8) {
                        float kv[8];
                        ld8(kc + (long)keys.at(j) * w.dp + c, kv);
#pragma unroll
                        for (int r = 0; r < RB; ++r) {
                            const float* q = qs + (r0 + (r < nr ? r : 0)) * w.dp + c;
#pragma unroll
                            for (int v = 0; v < 8; ++v) dot[r] = fmaf(q[v], kv[v], dot[r]);
                        }
                    }
                for (int o = 1; o < LPK; o <<= 1)
#pragma unroll
                    for (int r = 0; r < RB; ++r) dot[r] += __shfl_xor(dot[r], o, 64);
                if (kl == 0) {
#pragma unroll
                    for (int r = 0; r < RB; ++r) {
                        const int h = g * R + r0 + (r < nr ? r : 0);
                        ps[r * DK + kk] = j < k1 ? Score<SC>(a.sc, h).exact(dot[r], (float)(i - keys.at(j))) : -INFINITY;
                    }
                }
            }
            __syncthreads();
            for (int r = wave; r < RB; r += 4) {
                const float s = ps[r * DK + lane];
                const float mo = st[r * 4], mn = fmaxf(mo, wave_max(s));
                const float e = exp2f(s - mn);
                ps[r * DK + lane] = e;
                const float sum = wave_sum(e);
                if (lane == 0) {
                    const float al = exp2f(mo - mn);
                    st[r * 4] = mn;
                    st[r * 4 + 1] = st[r * 4 + 1] * al + sum;
                    st[r * 4 + 2] = al;
                }
            }
            __syncthreads();
#pragma unroll
            for (int r = 0; r < RB; ++r) {
                const float al = st[r * 4 + 2];
#pragma unroll
                for (int v = 0; v < 8; ++v) acc[r][v] *= al;
            }
            if (vch < nch) {
                const int n = min(DK, k1 - j0);
                for (int kk = vk; kk < n; kk += vkn) {
                    float vv[8];
                    ld8(vc + (long)keys.at(j0 + kk) * w.ep + vch * 8, vv);
#pragma unroll
                    for (int r = 0; r < RB; ++r) {
                        const float p = ps[r * DK + kk];
#pragma unroll
                        for (int v = 0; v < 8; ++v) acc[r][v] = fmaf(p, vv[v], acc[r][v]);
                    }
                }
            }
            __syncthreads();
        }
#pragma unroll
        for (int r = 0; r < RB; ++r) {
            if (r < nr) {
#pragma unroll
                for (int v = 0; v < 8; ++v) red[tid * 8 + v] = acc[r][v];
                __syncthreads();
                float* pr = part + (long)(r0 + r) * a.nsplit * rs;
                for (int c = tid; c < w.ep; c += 256) {
                    float t = 0.0f;
                    for (int k = 0; k < vkn; ++k) t += red[(k * CPV + c / 8) * 8 + c % 8];
                    pr[c] = t;
                }
                if (tid == 0) {
                    pr[w.ep] = st[r * 4];
                    pr[w.ep + 1] = st[r * 4 + 1];
                }
                __syncthreads();
            }
        }
    }
}

// bf16 MFMA form, 16 query heads of a group per workgroup (grid (split, G * head blocks, B)).  A wave takes 32-key
// tiles: S^T = K Q^T with the key fragments straight from the cache, then O^T += V^T P^T as k_wattn_m, the values
// through the wave's own LDS rows; the four waves' running sums meet in LDS.
template <int DQ, int DV, int SC>
__global__ void __launch_bounds__(256) k_wattn_dm(WAttnDecodeArgs a) {
    const WAttnHeads& w = a.hd;
    constexpr int VS = DV + 8;
    __shared__ __attribute__((aligned(16))) uint16_t Vs[4][32 * VS];
    __shared__ float sml[4][16][2];
    const int R = w.H / w.G, hb = blockIdx.y / w.G, g = blockIdx.y % w.G, b = blockIdx.z, sp = blockIdx.x;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, lg = lane >> 4;
    const int slot = a.slot[b], i = a.pos[b];
    const Keys keys(a.sc, i);  // k0, k1, kend, j0 below count the keys this query sees
    const int per = ((keys.n + a.nsplit - 1) / a.nsplit + 127) / 128 * 128;
    const int k0 = sp * per, k1 = min(keys.n, k0 + per);
    const uint16_t* qkv = reinterpret_cast<const uint16_t*>(a.qkv) + (long)b * a.ldqkv;
    const int r0 = hb * 16, nr = min(16, R - r0), rs = w.ep + 2;
    float* part = a.part + (((long)b * w.H + g * R + r0) * a.nsplit + sp) * rs;
    if (k0 >= k1) {
        if (tid < nr) {
            part[(long)tid * a.nsplit * rs + w.ep] = kNone;
            part[(long)tid * a.nsplit * rs + w.ep + 1] = 0.0f;
        }
        return;
    }
    uint16_t* kc = reinterpret_cast<uint16_t*>(a.kc) + ((long)slot * w.G + g) * a.max_tokens * w.dp;
    uint16_t* vc = reinterpret_cast<uint16_t*>(a.vc) + ((long)slot * w.G + g) * a.max_tokens * w.ep;
    // A new key (position i) never passes through the cache here: its score and value come from its qkv row, in
    // wave 0 of the last split, which also writes its cache rows.  Cached keys end at kend.
    const bool own = w.own_kv && k1 == keys.n;
    const int kend = own ? k1 - 1 : k1;
    const int h = g * R + r0 + (li < nr ? li : 0);
    const uint16_t* kn = qkv + w.H * w.d + g * w.d;
    const uint16_t* vn = qkv + (w.H + w.G) * w.d + g * w.e;
    // first tile's loads, then the query's: all in flight together
    uint4 vr[DV / 16], kr[2][DQ / 32];
    auto gload = [&](int j0) {
        const int jm = max(kend - 1, 0);
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            const uint16_t* p = kc + (long)keys.at(min(j0 + t * 16 + li, jm)) * w.dp;
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c) kr[t][c] = ldg16_sel(p + c * 32 + 8 * lg, c * 32 + 8 * lg < w.dp, p);
        }
#pragma unroll
        for (int x = 0; x < DV / 16; ++x) {
            const int e = lane + 64 * x, r = e / (DV / 8), k = (e % (DV / 8)) * 8;
            vr[x] = ldg16_sel(vc + (long)keys.at(min(j0 + r, jm)) * w.ep + k, k < w.ep, vc);
        }
    };
    if (k0 + wave * 32 < kend) gload(k0 + wave * 32);
    // a q or k head row's dims 8 lg .. 8 lg + 7 of every 32, normed and rotated, as bf16
    auto head_row = [&](const uint16_t* src, short8 (&f)[DQ / 32]) {
        float q[DQ / 32][8], ss = 0.0f;
        if (w.d % 8 == 0) {
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c) {
                const int k = c * 32 + 8 * lg;
                ld8(src + (k < w.d ? k : 0), q[c]);
#pragma unroll
                for (int v = 0; v < 8; ++v) q[c][v] = k < w.d ? q[c][v] : 0.0f;
            }
        } else {
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c)
#pragma unroll
                for (int v = 0; v < 8; ++v) {
                    const int k = c * 32 + 8 * lg + v;
                    q[c][v] = k < w.d ? bf2f(src[k]) : 0.0f;
                }
        }
        float inv = 1.0f;
        if (w.qk_norm) {
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c)
#pragma unroll
                for (int v = 0; v < 8; ++v) ss = fmaf(q[c][v], q[c][v], ss);
            ss += __shfl_xor(ss, 16, 64);
            ss += __shfl_xor(ss, 32, 64);
            inv = 1.0f / sqrtf(ss / (float)w.d + w.eps);
        }
#pragma unroll
        for (int c = 0; c < DQ / 32; ++c)
#pragma unroll
            for (int v = 0; v < 8; v += 2) {
                float x = q[c][v] * inv, y = q[c][v + 1] * inv;
                const int k = c * 32 + 8 * lg + v;
                if (k < w.rot) rotate(w.turns, k / 2, i, x, y);
                f[c][v] = (short)f2bf(x);
                f[c][v + 1] = (short)f2bf(y);
            }
    };
    short8 qf[DQ / 32];
    head_row(qkv + h * w.d, qf);
    const Score<SC> score(a.sc, h);
    f32x4 o[DV / 16];
#pragma unroll
    for (int c = 0; c < DV / 16; ++c) o[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = SC == SC_CAPPED ? 0.0f : kNone, l = 0.0f;
    if (own && wave == 0) {
        short8 kf[DQ / 32];
        head_row(kn, kf);
        float dot = 0.0f;
#pragma unroll
        for (int c = 0; c < DQ / 32; ++c)
#pragma unroll
            for (int v = 0; v < 8; ++v) dot = fmaf(bf2f((uint16_t)qf[c][v]), bf2f((uint16_t)kf[c][v]), dot);
        dot += __shfl_xor(dot, 16, 64);
        dot += __shfl_xor(dot, 32, 64);
        const float s = score.fast(dot, 0.0f);
        float p = 1.0f;
        if constexpr (SC == SC_CAPPED) p = __builtin_amdgcn_exp2f(s);
        else m = s;
        l = lg == 0 ? p : 0.0f;  // summed over the lane groups below
        const bool vec = w.d % 8 == 0 && w.e % 8 == 0;
        float vss = 0.0f;
#pragma unroll
        for (int c = 0; c < DV / 16; ++c) {
            const int k = c * 16 + 4 * lg;
            float v[4];
            if (vec) {
                ld4(vn + (k < w.e ? k : 0), v);
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] = k < w.e ? v[r] : 0.0f;
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] = k + r < w.e ? bf2f(vn[k + r]) : 0.0f;
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                o[c][r] = v[r];
                vss = fmaf(v[r], v[r], vss);
            }
        }
        float vinv = 1.0f;
        if (w.v_norm) {
            vss += __shfl_xor(vss, 16, 64);
            vss += __shfl_xor(vss, 32, 64);
            vinv = 1.0f / sqrtf(vss / (float)w.e + w.eps);
        }
#pragma unroll
        for (int c = 0; c < DV / 16; ++c)
#pragma unroll
            for (int r = 0; r < 4; ++r) o[c][r] = rbf(o[c][r] * vinv) * p;
        if (li == 0) {
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c)
                if (c * 32 + 8 * lg < w.dp) *reinterpret_cast<short8*>(kc + (long)i * w.dp + c * 32 + 8 * lg) = kf[c];
        }
        for (int k = lane; k < w.ep; k += 64) vc[(long)i * w.ep + k] = k < w.e ? f2bf(bf2f(vn[k]) * vinv) : 0;
    }
    for (int j0 = k0 + wave * 32; j0 < kend; j0 += 128) {
        f32x4 st[2];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            st[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c) st[t] = mfma16(__builtin_bit_cast(short8, kr[t][c]), qf[c], st[t]);
        }
        float mt = m;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int j = j0 + t * 16 + 4 * lg + r;
                const float s = score.fast(st[t][r], SC == SC_BIAS ? (float)(i - keys.at(j)) : 0.0f);
                st[t][r] = j < kend ? s : -INFINITY;
                if constexpr (SC != SC_CAPPED) mt = fmaxf(mt, st[t][r]);
            }
        float alpha = 1.0f;
        if constexpr (SC != SC_CAPPED) {
            mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
            mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
            alpha = __builtin_amdgcn_exp2f(m - mt);
            m = mt;
            l *= alpha;
        }
        short8 pf;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float p = __builtin_amdgcn_exp2f(st[t][r] - m);
                l += p;
                pf[4 * t + r] = (short)f2bf(p);
            }
#pragma unroll
        for (int x = 0; x < DV / 16; ++x) {
            const int e = lane + 64 * x, r = e / (DV / 8), k = (e % (DV / 8)) * 8;
            *reinterpret_cast<uint4*>(&Vs[wave][r * VS + k]) = vr[x];
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // this wave's own rows: no barrier
        if (j0 + 128 < kend) gload(j0 + 128);
#pragma unroll
        for (int c = 0; c < DV / 16; ++c) {
            if constexpr (SC != SC_CAPPED) {
#pragma unroll
                for (int r = 0; r < 4; ++r) o[c][r] *= alpha;
            }
            uint16_t* vp = &Vs[wave][(4 * lg + (li >> 2)) * VS + c * 16 + 4 * (li & 3)];
            const s4v lo4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(vp));
            const s4v hi4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4v*)(vp + 16 * VS));
            const short8 vf = {lo4[0], lo4[1], lo4[2], lo4[3], hi4[0], hi4[1], hi4[2], hi4[3]};
            o[c] = mfma16(vf, pf, o[c]);
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (lg == 0) { sml[wave][li][0] = m; sml[wave][li][1] = l; }
    __syncthreads();
    float M = kNone;
#pragma unroll
    for (int w = 0; w < 4; ++w) M = fmaxf(M, sml[w][li][0]);
    const float f = __builtin_amdgcn_exp2f(m - M);
    float* os = reinterpret_cast<float*>(&Vs[0][0]);  // [wave][head][DV + 4], in place of the value rows
    constexpr int OS = DV + 4;
    static_assert(4 * 16 * OS * 4 <= 4 * 32 * VS * 2, "the sums fit the value rows");
#pragma unroll
    for (int c = 0; c < DV / 16; ++c)
        *reinterpret_cast<float4*>(os + (wave * 16 + li) * OS + c * 16 + 4 * lg) =
            make_float4(o[c][0] * f, o[c][1] * f, o[c][2] * f, o[c][3] * f);
    __syncthreads();
    for (int e = tid; e < nr * w.ep; e += 256) {
        const int r = e / w.ep, c = e % w.ep;
        float t = 0.0f;
#pragma unroll
        for (int w = 0; w < 4; ++w) t += os[(w * 16 + r) * OS + c];
        part[(long)r * a.nsplit * rs + c] = t;
    }
    if (tid < nr) {
        float mm = kNone, ll = 0.0f;
#pragma unroll
        for (int w = 0; w < 4; ++w) mm = fmaxf(mm, sml[w][tid][0]);
#pragma unroll
        for (int w = 0; w < 4; ++w) ll += sml[w][tid][1] * __builtin_amdgcn_exp2f(sml[w][tid][0] - mm);
        part[(long)tid * a.nsplit * rs + w.ep] = mm;
        part[(long)tid * a.nsplit * rs + w.ep + 1] = ll;
    }
}

// merge a head's partials: grid (H, B), nsplit <= 64
template <typename T>
__global__ void __launch_bounds__(256) k_wattn_dc(WAttnDecodeArgs a) {
    __shared__ float wt[64];
    const int h = blockIdx.x, b = blockIdx.y, rs = a.hd.ep + 2, n = a.nsplit, lane = threadIdx.x & 63;
    const float* p = a.part + ((long)b * a.hd.H + h) * n * rs;
    {
        const float m = lane < n ? p[(long)lane * rs + a.hd.ep] : kNone, l = lane < n ? p[(long)lane * rs + a.hd.ep + 1] : 0.0f;
        const float M = wave_max(l > 0.0f ? m : kNone);
        const float w = l > 0.0f ? exp2f(m - M) : 0.0f;
        const float L = wave_sum(l * w);
        if (threadIdx.x < 64) wt[lane] = w / L;
    }
    __syncthreads();
    T* o = reinterpret_cast<T*>(a.o) + (long)b * a.ldo;
    for (int c = threadIdx.x; c < a.hd.e; c += 256) {
        float t = 0.0f;
        // an empty split's values were never written: weight 0, not read
#pragma unroll 8
        for (int s = 0; s < n; ++s)
            if (wt[s] > 0.0f) t = fmaf(p[(long)s * rs + c], wt[s], t);
        stf(o + h * a.hd.e + c, t);
    }
    if (h == a.hd.H - 1)
        for (int k = a.hd.H * a.hd.e + threadIdx.x; k < a.ldo; k += 256) stf(o + k, 0.0f);
}

template <typename T, int RB, int SC>
void run_d(hipStream_t s, const WAttnDecodeArgs& a) {
    const WAttnHeads& w = a.hd;
    const size_t lds = (size_t)(w.H / w.G * w.dp + RB * DK + RB * 4 + 256 * 8) * sizeof(float);
    if (lds > 64 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&k_wattn_d<T, RB, SC>),
                                  hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL((k_wattn_d<T, RB, SC>), dim3(a.nsplit, w.G, a.B), dim3(256), lds, s, a);
    hipLaunchKernelGGL((k_wattn_dc<T>), dim3(w.H, a.B), dim3(256), 0, s, a);
}

template <int DQ, int DV>
void run_dm(hipStream_t s, const WAttnDecodeArgs& a) {
    const WAttnHeads& w = a.hd;
    const dim3 grid(a.nsplit, w.G * ((w.H / w.G + 15) / 16), a.B);
    const int mode = score_mode(a.sc);
    if (mode == SC_BIAS) hipLaunchKernelGGL((k_wattn_dm<DQ, DV, SC_BIAS>), grid, dim3(256), 0, s, a);
    else if (mode == SC_CAPPED) hipLaunchKernelGGL((k_wattn_dm<DQ, DV, SC_CAPPED>), grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((k_wattn_dm<DQ, DV, SC_PLAIN>), grid, dim3(256), 0, s, a);
    hipLaunchKernelGGL((k_wattn_dc<uint16_t>), dim3(w.H, a.B), dim3(256), 0, s, a);
}
template <int DQ>
void run_dmv(hipStream_t s, const WAttnDecodeArgs& a) {
    if (a.hd.ep <= 64) run_dm<DQ, 64>(s, a);
    else if (a.hd.ep <= 128) run_dm<DQ, 128>(s, a);
    else run_dm<DQ, 256>(s, a);
}

template <typename T, int SC>
void decode_sc(hipStream_t s, const WAttnDecodeArgs& a) {
    const int R = a.hd.H / a.hd.G;
    if (R <= 1) run_d<T, 1, SC>(s, a);
    else if (R <= 2) run_d<T, 2, SC>(s, a);
    else if (R <= 4) run_d<T, 4, SC>(s, a);
    else run_d<T, 8, SC>(s, a);
}
template <typename T>
void decode_t(hipStream_t s, const WAttnDecodeArgs& a) {
    if (a.sc.r1) decode_sc<T, SC_BIAS>(s, a);
    else decode_sc<T, SC_PLAIN>(s, a);
}

template <typename T>
void plain_t(hipStream_t s, const WAttnArgs& a) {
    const size_t lds = (size_t)(a.hd.dp + 256 + 8) * sizeof(float);
    const dim3 grid(a.rows, a.hd.H);
    if (a.sc.r1) hipLaunchKernelGGL((k_wattn<T, SC_BIAS>), grid, dim3(256), lds, s, a);
    else hipLaunchKernelGGL((k_wattn<T, SC_PLAIN>), grid, dim3(256), lds, s, a);
}

}  // namespace

void wattn_append(hipStream_t s, Act act, const WAttnArgs& a) {
    if (act == ACT_F32) append_t<float>(s, a);
    else append_t<uint16_t>(s, a);
}

void wattn_prefill(hipStream_t s, Act act, const WAttnArgs& a) {
    const int dp = a.hd.dp, ep = a.hd.ep;
    if (act == ACT_F32) {
        plain_t<float>(s, a);
    } else if (dp > 256 || ep > 256) {
        plain_t<uint16_t>(s, a);
    } else if (dp <= 64) {
        run_mv<64>(s, a);
    } else if (dp <= 96) {
        run_mv<96>(s, a);
    } else if (dp <= 128) {
        run_mv<128>(s, a);
    } else {
        run_mv<256>(s, a);
    }
}

int wattn_decode_splits(int B, int G, const WAttnScore& sc, int max_tokens) {
    const int span = (int)std::max(1L, std::min((long)sc.window + sc.keep, (long)max_tokens));
    const int tiles = (span + 127) / 128;
    int n = (1024 + B * G - 1) / (B * G);
    return std::max(1, std::min(std::min(n, tiles), 64));
}

size_t wattn_decode_floats(int B, int H, int ep, int nsplit) { return (size_t)B * H * nsplit * (ep + 2); }

void wattn_decode(hipStream_t s, Act act, const WAttnDecodeArgs& a) {
    const int dp = a.hd.dp, ep = a.hd.ep;
    if (act == ACT_F32) decode_t<float>(s, a);
    else if (dp > 256 || ep > 256) decode_t<uint16_t>(s, a);
    else if (dp <= 64) run_dmv<64>(s, a);
    else if (dp <= 128) run_dmv<128>(s, a);
    else run_dmv<256>(s, a);
}

}  // namespace pgmi
