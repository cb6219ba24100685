// kernels_wattn.hip -- grouped-query attention over a sliding window with a logarithmic distance bias, query and
// key heads over their root mean squares, any head sizes.  Scores, weights and norms are fp32.
//
//   k_append    norms q and k of a prefill's rows, writes the key / value rows into the cache
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

// score in powers of two: dot * c1 - r1 log2(1 + r2 dist)
__device__ __forceinline__ float biased(float dot, float c1, float r1, float r2, float dist) {
    return dot * c1 - r1 * __builtin_amdgcn_logf(fmaf(r2, dist, 1.0f));
}
// fp32 activations: the library logarithm
__device__ __forceinline__ float biased_exact(float dot, float c1, float r1, float r2, float dist) {
    return dot * c1 - r1 * (log1pf(r2 * dist) * kLog2e);
}

// ---------------------------------------------------------------- append
// LPH lanes per head of a row (8 elements each when V == 8: head sizes that are multiples of 8)
template <typename T, int LPH, int V>
__global__ void __launch_bounds__(256) k_append(WAttnArgs a) {
    const int row = blockIdx.x, sub = threadIdx.x % LPH;
    const int head = blockIdx.y * (256 / LPH) + threadIdx.x / LPH, NH = a.H + 2 * a.G;
    const SeqInfo q = a.seqs[a.row_seq[row]];
    const long pos = q.start + (row - q.off);
    const T* src = reinterpret_cast<const T*>(a.qkv) + (long)row * a.ldqkv;
    const int hd = head < NH ? head : NH - 1;
    T* dst;
    int n, np;
    const bool norm = hd < a.H + a.G;
    if (hd < a.H) {
        src += hd * a.d; n = a.d; np = a.dp;
        dst = reinterpret_cast<T*>(a.q) + ((long)row * a.H + hd) * a.dp;
    } else if (hd < a.H + a.G) {
        const int g = hd - a.H;
        src += a.H * a.d + g * a.d; n = a.d; np = a.dp;
        dst = reinterpret_cast<T*>(a.kc) + (((long)q.slot * a.G + g) * a.max_tokens + pos) * a.dp;
    } else {
        const int g = hd - a.H - a.G;
        src += (a.H + a.G) * a.d + g * a.e; n = a.e; np = a.ep;
        dst = reinterpret_cast<T*>(a.vc) + (((long)q.slot * a.G + g) * a.max_tokens + pos) * a.ep;
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
    const float inv = norm ? 1.0f / sqrtf(ss / (float)n + a.eps) : 1.0f;
    if (head >= NH) return;
    for (int i = sub * V; i < np; i += LPH * V) {
        if constexpr (V == 8) {
            float v[8];
            ld8(src + i, v);
#pragma unroll
            for (int t = 0; t < 8; ++t) v[t] *= inv;
            st8(dst + i, v);
        } else {
            stf(dst + i, i < n ? ldf(src + i) * inv : 0.0f);
        }
    }
}

template <typename T>
void append_t(hipStream_t s, const WAttnArgs& a) {
    const int NH = a.H + 2 * a.G;
    if (a.d % 8 == 0 && a.e % 8 == 0)
        hipLaunchKernelGGL((k_append<T, 16, 8>), dim3(a.rows, (NH + 15) / 16), dim3(256), 0, s, a);
    else
        hipLaunchKernelGGL((k_append<T, 64, 1>), dim3(a.rows, (NH + 3) / 4), dim3(256), 0, s, a);
}

// ---------------------------------------------------------------- plain form
template <typename T>
__global__ void __launch_bounds__(256) k_wattn(WAttnArgs a) {
    extern __shared__ float sm[];
    float* qs = sm;              // [dp]
    float* p = qs + a.dp;        // [256]
    float* red = p + 256;        // [8]
    const int row = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const SeqInfo q = a.seqs[a.row_seq[row]];
    const int i = q.start + (row - q.off), g = h / (a.H / a.G);
    const T* qp = reinterpret_cast<const T*>(a.q) + ((long)row * a.H + h) * a.dp;
    for (int k = tid; k < a.dp; k += 256) qs[k] = ldf(qp + k);
    __syncthreads();
    const T* kc = reinterpret_cast<const T*>(a.kc) + ((long)q.slot * a.G + g) * a.max_tokens * a.dp;
    const T* vc = reinterpret_cast<const T*>(a.vc) + ((long)q.slot * a.G + g) * a.max_tokens * a.ep;
    const float r1 = bf2f(a.r1[h]), r2 = bf2f(a.r2[h]), c1 = a.scale * kLog2e;
    const int lo = max(0, i - a.window + 1);
    float m = kNone, l = 0.0f;
    constexpr int EM = 8;  // value columns per thread: e <= 2048
    float acc[EM] = {};
    for (int j0 = lo; j0 <= i; j0 += 256) {
        const int j = j0 + tid;
        float s = -INFINITY;
        if (j <= i) {
            const T* kr = kc + (long)j * a.dp;
            float dot = 0.0f;
            for (int k = 0; k < a.d; ++k) dot = fmaf(qs[k], ldf(kr + k), dot);
            s = biased_exact(dot, c1, r1, r2, (float)(i - j));
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
        const int n = min(256, i - j0 + 1);
#pragma unroll
        for (int v = 0; v < EM; ++v) {
            const int col = tid + 256 * v;
            if (col < a.e) {
                float o = acc[v] * alpha;
                for (int k = 0; k < n; ++k) o = fmaf(p[k], ldf(vc + (long)(j0 + k) * a.ep + col), o);
                acc[v] = o;
            }
        }
        __syncthreads();
    }
    T* o = reinterpret_cast<T*>(a.o) + (long)row * a.ldo;
#pragma unroll
    for (int v = 0; v < EM; ++v) {
        const int col = tid + 256 * v;
        if (col < a.e) stf(o + h * a.e + col, acc[v] / l);
    }
    if (h == a.H - 1)
        for (int k = a.H * a.e + tid; k < a.ldo; k += 256) stf(o + k, 0.0f);
}

// ---------------------------------------------------------------- bf16 MFMA form
// Scores are computed transposed, S^T = K Q^T, so that a lane holds one query row (column lane & 15) and, after
// two 16-key tiles, exactly the 8 weights its B fragment of O^T = V^T P^T needs (the contraction order is free:
// slot 8g + i is key 4g + i of the first tile for i < 4, of the second for i >= 4).  V^T fragments are
// transposed LDS reads of the row-major V tile.
template <int DQ, int DV>
__global__ void __launch_bounds__(256) k_wattn_m(WAttnArgs a) {
    constexpr int KT = 64;                 // keys per tile
    constexpr int KS = DQ + 8, VS = DV + 8;  // LDS row strides (elements)
    constexpr int KQ = KT * DQ / 8 / 256, VQ = KT * DV / 8 / 256;  // 16-byte pieces per thread
    __shared__ __attribute__((aligned(16))) uint16_t Ks[KT * KS];
    __shared__ __attribute__((aligned(16))) uint16_t Vs[KT * VS];
    const ChunkInfo tl = a.tiles[blockIdx.x];
    const SeqInfo sq = a.seqs[tl.seq];
    const int g = blockIdx.y, R = a.H / a.G;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane & 15, lg = lane >> 4;
    const int nrow = sq.len * R;
    // this lane's query row
    const int fr = tl.rel + wave * 16 + li;
    const bool ok = fr < nrow;
    const int frc = ok ? fr : nrow - 1;
    const int prow = frc / R, hh = frc % R, h = g * R + hh;
    const int i = sq.start + prow;
    const uint16_t* qp = reinterpret_cast<const uint16_t*>(a.q) + ((long)(sq.off + prow) * a.H + h) * a.dp;
    short8 qf[DQ / 32];
#pragma unroll
    for (int c = 0; c < DQ / 32; ++c) {
        const int k = c * 32 + 8 * lg;
        const uint4 v = ldg16_sel(qp + k, k < a.dp, qp);
        qf[c] = __builtin_bit_cast(short8, v);
    }
    const float r1 = bf2f(a.r1[h]), r2 = bf2f(a.r2[h]), c1 = a.scale * kLog2e;
    // keys the tile's rows see: [lo, hi]
    const int last = min(tl.rel + kWAttnRows, nrow) - 1;
    const int lo = max(0, sq.start + tl.rel / R - a.window + 1), hi = sq.start + last / R;
    // positions of this wave's first and last rows
    const int wfirst = sq.start + min(tl.rel + wave * 16, nrow - 1) / R;
    const int wlast = sq.start + min(tl.rel + wave * 16 + 15, nrow - 1) / R;
    const uint16_t* kc = reinterpret_cast<const uint16_t*>(a.kc) + ((long)sq.slot * a.G + g) * a.max_tokens * a.dp;
    const uint16_t* vc = reinterpret_cast<const uint16_t*>(a.vc) + ((long)sq.slot * a.G + g) * a.max_tokens * a.ep;
    f32x4 o[DV / 16];
#pragma unroll
    for (int c = 0; c < DV / 16; ++c) o[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = kNone, l = 0.0f;
    uint4 kr[KQ], vr[VQ];
    auto gload = [&](int j0) {
#pragma unroll
        for (int x = 0; x < KQ; ++x) {
            const int e = tid + 256 * x, r = e / (DQ / 8), k = (e % (DQ / 8)) * 8;
            const int j = min(j0 + r, hi);
            kr[x] = ldg16_sel(kc + (long)j * a.dp + k, k < a.dp, kc);
        }
#pragma unroll
        for (int x = 0; x < VQ; ++x) {
            const int e = tid + 256 * x, r = e / (DV / 8), k = (e % (DV / 8)) * 8;
            const int j = min(j0 + r, hi);
            vr[x] = ldg16_sel(vc + (long)j * a.ep + k, k < a.ep, vc);
        }
    };
    gload(lo);
    for (int j0 = lo; j0 <= hi; j0 += KT) {
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
        if (j0 + KT <= hi) gload(j0 + KT);
        if (j0 > wlast || j0 + KT <= wfirst - a.window + 1) continue;  // no row of this wave sees the tile
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
        float mt = m;
        // 1 + r2 (i - j) for key j0 + 4 lg, less r2 per key after it
        const float x0 = fmaf(r2, (float)(i - j0 - 4 * lg), 1.0f);
        if (j0 + KT - 1 <= wfirst && wlast - j0 < a.window) {  // every row sees every key
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float x = fmaf(-r2, (float)(t * 16 + r), x0);
                    st[t][r] = fmaf(-r1, __builtin_amdgcn_logf(x), st[t][r] * c1);
                    mt = fmaxf(mt, st[t][r]);
                }
        } else {
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int dist = i - (j0 + t * 16 + 4 * lg + r);
                    const float x = fmaf(-r2, (float)(t * 16 + r), x0);
                    const float s = fmaf(-r1, __builtin_amdgcn_logf(x), st[t][r] * c1);
                    st[t][r] = (unsigned)dist < (unsigned)a.window ? s : -INFINITY;
                    mt = fmaxf(mt, st[t][r]);
                }
        }
        mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
        mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
        const float alpha = __builtin_amdgcn_exp2f(m - mt);
        m = mt;
        float ls = 0.0f;
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                st[t][r] = __builtin_amdgcn_exp2f(st[t][r] - m);
                ls += st[t][r];
            }
        l = l * alpha + ls;  // this lane's keys; summed over the lane groups at the end
        if (__any(alpha != 1.0f)) {
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
    uint16_t* op = reinterpret_cast<uint16_t*>(a.o) + (long)(sq.off + prow) * a.ldo + h * a.e;
#pragma unroll
    for (int c = 0; c < DV / 16; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int col = c * 16 + 4 * lg + r;
            if (col < a.e) op[col] = f2bf(o[c][r] * inv);
        }
    if (h == a.H - 1 && lg == 0)
        for (int k = a.H * a.e; k < a.ldo; ++k) reinterpret_cast<uint16_t*>(a.o)[(long)(sq.off + prow) * a.ldo + k] = 0;
}

template <int DQ, int DV>
void run_m(hipStream_t s, const WAttnArgs& a) {
    hipLaunchKernelGGL((k_wattn_m<DQ, DV>), dim3(a.ntile, a.G), dim3(256), 0, s, a);
}
template <int DQ>
void run_mv(hipStream_t s, const WAttnArgs& a) {
    if (a.ep <= 64) run_m<DQ, 64>(s, a);
    else if (a.ep <= 96) run_m<DQ, 96>(s, a);
    else if (a.ep <= 128) run_m<DQ, 128>(s, a);
    else run_m<DQ, 256>(s, a);
}

// ---------------------------------------------------------------- one token per sequence
constexpr int DK = 64;  // keys per tile

// grid (split, G, B).  RB: query heads of the group handled at once (registers).
// part record of (b, head, split): [ep] weighted values, then running maximum, then sum of weights
template <typename T, int RB>
__global__ void __launch_bounds__(256) k_wattn_d(WAttnDecodeArgs a) {
    extern __shared__ float sm[];
    const int R = a.H / a.G;
    float* qs = sm;                 // [R][dp] normalised queries
    float* ps = qs + R * a.dp;      // [RB][DK] scores, then weights
    float* st = ps + RB * DK;       // [RB][4]: running max, sum, alpha
    float* red = st + RB * 4;       // [256][8] cross-group reduction
    const int g = blockIdx.y, b = blockIdx.z, sp = blockIdx.x;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int slot = a.slot[b], i = a.pos[b];
    const int lo = max(0, i - a.window + 1), span = i - lo + 1;
    const int per = ((span + a.nsplit - 1) / a.nsplit + DK - 1) / DK * DK;
    const int k0 = lo + sp * per, k1 = min(i + 1, k0 + per);  // empty when k0 >= k1
    const T* qkv = reinterpret_cast<const T*>(a.qkv) + (long)b * a.ldqkv;
    const int rs = a.ep + 2;
    float* part = a.part + (((long)b * a.H + g * R) * a.nsplit + sp) * rs;
    if (k0 >= k1) {
        for (int r = tid; r < R; r += 256) {
            part[(long)r * a.nsplit * rs + a.ep] = kNone;
            part[(long)r * a.nsplit * rs + a.ep + 1] = 0.0f;
        }
        return;
    }
    T* kc = reinterpret_cast<T*>(a.kc) + ((long)slot * a.G + g) * a.max_tokens * a.dp;
    T* vc = reinterpret_cast<T*>(a.vc) + ((long)slot * a.G + g) * a.max_tokens * a.ep;
    for (int r = wave; r < R; r += 4) {
        const T* src = qkv + (g * R + r) * a.d;
        float ss = 0.0f;
        for (int k = lane; k < a.d; k += 64) ss = fmaf(ldf(src + k), ldf(src + k), ss);
        const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)a.d + a.eps);
        // queries rounded as the prefill form rounds them
        for (int k = lane; k < a.dp; k += 64) {
            T t;
            stf(&t, k < a.d ? ldf(src + k) * inv : 0.0f);
            qs[r * a.dp + k] = ldf(&t);
        }
    }
    if (k1 == i + 1) {  // this workgroup's keys include the new one: write its cache rows
        if (wave == 0) {
            const T* src = qkv + a.H * a.d + g * a.d;
            float ss = 0.0f;
            for (int k = lane; k < a.d; k += 64) ss = fmaf(ldf(src + k), ldf(src + k), ss);
            const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)a.d + a.eps);
            for (int k = lane; k < a.dp; k += 64) stf(kc + (long)i * a.dp + k, k < a.d ? ldf(src + k) * inv : 0.0f);
        } else if (wave == 1) {
            const T* src = qkv + (a.H + a.G) * a.d + g * a.e;
            for (int k = lane; k < a.ep; k += 64) stf(vc + (long)i * a.ep + k, k < a.e ? ldf(src + k) : 0.0f);
        }
        __threadfence_block();
    }
    __syncthreads();
    const float c1 = a.scale * kLog2e;
    // scores: LPK lanes share a key, 8 elements each per step
    int LPK = 1;
    while (LPK < 64 && LPK * 8 < a.dp) LPK <<= 1;
    const int kl = lane % LPK, kw = wave * (64 / LPK) + lane / LPK, kstep = 4 * (64 / LPK);
    // weighted values: CPV threads span the columns (8 each), the rest split the keys
    const int nch = a.ep / 8;
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
                    for (int c = kl * 8; c < a.dp; c += LPK * 8) {
                        float kv[8];
                        ld8(kc + (long)j * a.dp + c, kv);
#pragma unroll
                        for (int r = 0; r < RB; ++r) {
                            const float* q = qs + (r0 + (r < nr ? r : 0)) * a.dp + c;
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
                        ps[r * DK + kk] = j < k1 ? biased_exact(dot[r], c1, bf2f(a.r1[h]), bf2f(a.r2[h]), (float)(i - j))
                                                 : -INFINITY;
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
                    ld8(vc + (long)(j0 + kk) * a.ep + vch * 8, vv);
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
                for (int c = tid; c < a.ep; c += 256) {
                    float t = 0.0f;
                    for (int k = 0; k < vkn; ++k) t += red[(k * CPV + c / 8) * 8 + c % 8];
                    pr[c] = t;
                }
                if (tid == 0) {
                    pr[a.ep] = st[r * 4];
                    pr[a.ep + 1] = st[r * 4 + 1];
                }
                __syncthreads();
            }
        }
    }
}

// bf16 MFMA form, 16 query heads of a group per workgroup (grid (split, G * head blocks, B)).  A wave takes 32-key
// tiles: S^T = K Q^T with the key fragments straight from the cache, then O^T += V^T P^T as k_wattn_m, the values
// through the wave's own LDS rows; the four waves' running sums meet in LDS.
template <int DQ, int DV>
__global__ void __launch_bounds__(256) k_wattn_dm(WAttnDecodeArgs a) {
    constexpr int VS = DV + 8;
    __shared__ __attribute__((aligned(16))) uint16_t Vs[4][32 * VS];
    __shared__ float sml[4][16][2];
    const int R = a.H / a.G, hb = blockIdx.y / a.G, g = blockIdx.y % a.G, b = blockIdx.z, sp = blockIdx.x;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, lg = lane >> 4;
    const int slot = a.slot[b], i = a.pos[b];
    const int lo = max(0, i - a.window + 1), span = i - lo + 1;
    const int per = ((span + a.nsplit - 1) / a.nsplit + 127) / 128 * 128;
    const int k0 = lo + sp * per, k1 = min(i + 1, k0 + per);
    const uint16_t* qkv = reinterpret_cast<const uint16_t*>(a.qkv) + (long)b * a.ldqkv;
    const int r0 = hb * 16, nr = min(16, R - r0), rs = a.ep + 2;
    float* part = a.part + (((long)b * a.H + g * R + r0) * a.nsplit + sp) * rs;
    if (k0 >= k1) {
        if (tid < nr) {
            part[(long)tid * a.nsplit * rs + a.ep] = kNone;
            part[(long)tid * a.nsplit * rs + a.ep + 1] = 0.0f;
        }
        return;
    }
    uint16_t* kc = reinterpret_cast<uint16_t*>(a.kc) + ((long)slot * a.G + g) * a.max_tokens * a.dp;
    uint16_t* vc = reinterpret_cast<uint16_t*>(a.vc) + ((long)slot * a.G + g) * a.max_tokens * a.ep;
    // The new token (position i) never passes through the cache here: its score and value come from its qkv row, in
    // wave 0 of the last split, which also writes its cache rows.  Cached keys end at kend.
    const bool own = k1 == i + 1;
    const int kend = own ? i : k1;
    const int h = g * R + r0 + (li < nr ? li : 0);
    const uint16_t* kn = qkv + a.H * a.d + g * a.d;
    const uint16_t* vn = qkv + (a.H + a.G) * a.d + g * a.e;
    // first tile's loads, then the query's: all in flight together
    uint4 vr[DV / 16], kr[2][DQ / 32];
    auto gload = [&](int j0) {
        const int jm = max(kend - 1, 0);
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            const uint16_t* p = kc + (long)min(j0 + t * 16 + li, jm) * a.dp;
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c) kr[t][c] = ldg16_sel(p + c * 32 + 8 * lg, c * 32 + 8 * lg < a.dp, p);
        }
#pragma unroll
        for (int x = 0; x < DV / 16; ++x) {
            const int e = lane + 64 * x, r = e / (DV / 8), k = (e % (DV / 8)) * 8;
            vr[x] = ldg16_sel(vc + (long)min(j0 + r, jm) * a.ep + k, k < a.ep, vc);
        }
    };
    if (k0 + wave * 32 < kend) gload(k0 + wave * 32);
    // a head row's dims 8 lg .. 8 lg + 7 of every 32, over its root mean square, as bf16
    auto unit_row = [&](const uint16_t* src, short8 (&f)[DQ / 32]) {
        float q[DQ / 32][8], ss = 0.0f;
        if (a.d % 8 == 0) {
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c) {
                const int k = c * 32 + 8 * lg;
                ld8(src + (k < a.d ? k : 0), q[c]);
#pragma unroll
                for (int v = 0; v < 8; ++v) q[c][v] = k < a.d ? q[c][v] : 0.0f;
            }
        } else {
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c)
#pragma unroll
                for (int v = 0; v < 8; ++v) {
                    const int k = c * 32 + 8 * lg + v;
                    q[c][v] = k < a.d ? bf2f(src[k]) : 0.0f;
                }
        }
#pragma unroll
        for (int c = 0; c < DQ / 32; ++c)
#pragma unroll
            for (int v = 0; v < 8; ++v) ss = fmaf(q[c][v], q[c][v], ss);
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        const float inv = 1.0f / sqrtf(ss / (float)a.d + a.eps);
#pragma unroll
        for (int c = 0; c < DQ / 32; ++c)
#pragma unroll
            for (int v = 0; v < 8; ++v) f[c][v] = (short)f2bf(q[c][v] * inv);
    };
    short8 qf[DQ / 32];
    unit_row(qkv + h * a.d, qf);
    const float r1 = bf2f(a.r1[h]), r2 = bf2f(a.r2[h]), c1 = a.scale * kLog2e;
    f32x4 o[DV / 16];
#pragma unroll
    for (int c = 0; c < DV / 16; ++c) o[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = kNone, l = 0.0f;
    if (own && wave == 0) {
        short8 kf[DQ / 32];
        unit_row(kn, kf);
        float dot = 0.0f;
#pragma unroll
        for (int c = 0; c < DQ / 32; ++c)
#pragma unroll
            for (int v = 0; v < 8; ++v) dot = fmaf(bf2f((uint16_t)qf[c][v]), bf2f((uint16_t)kf[c][v]), dot);
        dot += __shfl_xor(dot, 16, 64);
        dot += __shfl_xor(dot, 32, 64);
        m = dot * c1;  // distance 0: no bias; weight exp2(m - m) = 1
        l = lg == 0 ? 1.0f : 0.0f;  // summed over the lane groups below
        const bool vec = a.d % 8 == 0 && a.e % 8 == 0;
#pragma unroll
        for (int c = 0; c < DV / 16; ++c) {
            const int k = c * 16 + 4 * lg;
            float v[4];
            if (vec) {
                ld4(vn + (k < a.e ? k : 0), v);
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] = k < a.e ? v[r] : 0.0f;
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] = k + r < a.e ? bf2f(vn[k + r]) : 0.0f;
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) o[c][r] = v[r];
        }
        if (li == 0) {
#pragma unroll
            for (int c = 0; c < DQ / 32; ++c)
                if (c * 32 + 8 * lg < a.dp) *reinterpret_cast<short8*>(kc + (long)i * a.dp + c * 32 + 8 * lg) = kf[c];
        }
        for (int k = lane; k < a.ep; k += 64) vc[(long)i * a.ep + k] = k < a.e ? vn[k] : 0;
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
                st[t][r] = j < kend ? biased(st[t][r], c1, r1, r2, (float)(i - j)) : -INFINITY;
                mt = fmaxf(mt, st[t][r]);
            }
        mt = fmaxf(mt, __shfl_xor(mt, 16, 64));
        mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
        const float alpha = __builtin_amdgcn_exp2f(m - mt);
        m = mt;
        l *= alpha;
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
#pragma unroll
            for (int r = 0; r < 4; ++r) o[c][r] *= alpha;
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
    for (int e = tid; e < nr * a.ep; e += 256) {
        const int r = e / a.ep, c = e % a.ep;
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
        part[(long)tid * a.nsplit * rs + a.ep] = mm;
        part[(long)tid * a.nsplit * rs + a.ep + 1] = ll;
    }
}

// merge a head's partials: grid (H, B), nsplit <= 64
template <typename T>
__global__ void __launch_bounds__(256) k_wattn_dc(WAttnDecodeArgs a) {
    __shared__ float wt[64];
    const int h = blockIdx.x, b = blockIdx.y, rs = a.ep + 2, n = a.nsplit, lane = threadIdx.x & 63;
    const float* p = a.part + ((long)b * a.H + h) * n * rs;
    {
        const float m = lane < n ? p[(long)lane * rs + a.ep] : kNone, l = lane < n ? p[(long)lane * rs + a.ep + 1] : 0.0f;
        const float M = wave_max(l > 0.0f ? m : kNone);
        const float w = l > 0.0f ? exp2f(m - M) : 0.0f;
        const float L = wave_sum(l * w);
        if (threadIdx.x < 64) wt[lane] = w / L;
    }
    __syncthreads();
    T* o = reinterpret_cast<T*>(a.o) + (long)b * a.ldo;
    for (int c = threadIdx.x; c < a.e; c += 256) {
        float t = 0.0f;
        // an empty split's values were never written: weight 0, not read
#pragma unroll 8
        for (int s = 0; s < n; ++s)
            if (wt[s] > 0.0f) t = fmaf(p[(long)s * rs + c], wt[s], t);
        stf(o + h * a.e + c, t);
    }
    if (h == a.H - 1)
        for (int k = a.H * a.e + threadIdx.x; k < a.ldo; k += 256) stf(o + k, 0.0f);
}

template <typename T, int RB>
void run_d(hipStream_t s, const WAttnDecodeArgs& a) {
    const int R = a.H / a.G;
    const size_t lds = (size_t)(R * a.dp + RB * DK + RB * 4 + 256 * 8) * sizeof(float);
    if (lds > 64 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&k_wattn_d<T, RB>),
                                  hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL((k_wattn_d<T, RB>), dim3(a.nsplit, a.G, a.B), dim3(256), lds, s, a);
    hipLaunchKernelGGL((k_wattn_dc<T>), dim3(a.H, a.B), dim3(256), 0, s, a);
}

template <int DQ, int DV>
void run_dm(hipStream_t s, const WAttnDecodeArgs& a) {
    hipLaunchKernelGGL((k_wattn_dm<DQ, DV>), dim3(a.nsplit, a.G * ((a.H / a.G + 15) / 16), a.B), dim3(256), 0, s, a);
    hipLaunchKernelGGL((k_wattn_dc<uint16_t>), dim3(a.H, a.B), dim3(256), 0, s, a);
}
template <int DQ>
void run_dmv(hipStream_t s, const WAttnDecodeArgs& a) {
    if (a.ep <= 64) run_dm<DQ, 64>(s, a);
    else if (a.ep <= 128) run_dm<DQ, 128>(s, a);
    else run_dm<DQ, 256>(s, a);
}

template <typename T>
void decode_t(hipStream_t s, const WAttnDecodeArgs& a) {
    const int R = a.H / a.G;
    if (R <= 1) run_d<T, 1>(s, a);
    else if (R <= 2) run_d<T, 2>(s, a);
    else if (R <= 4) run_d<T, 4>(s, a);
    else run_d<T, 8>(s, a);
}

template <typename T>
void plain_t(hipStream_t s, const WAttnArgs& a) {
    const size_t lds = (size_t)(a.dp + 256 + 8) * sizeof(float);
    hipLaunchKernelGGL((k_wattn<T>), dim3(a.rows, a.H), dim3(256), lds, s, a);
}

}  // namespace

void wattn_append(hipStream_t s, Act act, const WAttnArgs& a) {
    if (act == ACT_F32) append_t<float>(s, a);
    else append_t<uint16_t>(s, a);
}

void wattn_prefill(hipStream_t s, Act act, const WAttnArgs& a) {
    if (act == ACT_F32) {
        plain_t<float>(s, a);
    } else if (a.dp > 256 || a.ep > 256) {
        plain_t<uint16_t>(s, a);
    } else if (a.dp <= 64) {
        run_mv<64>(s, a);
    } else if (a.dp <= 96) {
        run_mv<96>(s, a);
    } else if (a.dp <= 128) {
        run_mv<128>(s, a);
    } else {
        run_mv<256>(s, a);
    }
}

int wattn_decode_splits(int B, int G, int window, int max_tokens) {
    const int span = std::max(1, std::min(window, max_tokens));
    const int tiles = (span + 127) / 128;
    int n = (1024 + B * G - 1) / (B * G);
    return std::max(1, std::min(std::min(n, tiles), 64));
}

size_t wattn_decode_floats(int B, int H, int ep, int nsplit) { return (size_t)B * H * nsplit * (ep + 2); }

void wattn_decode(hipStream_t s, Act act, const WAttnDecodeArgs& a) {
    if (act == ACT_F32) decode_t<float>(s, a);
    else if (a.dp > 256 || a.ep > 256) decode_t<uint16_t>(s, a);
    else if (a.dp <= 64) run_dmv<64>(s, a);
    else if (a.dp <= 128) run_dmv<128>(s, a);
    else run_dmv<256>(s, a);
}

}  // namespace pgmi
