// kernels_wattn.hip -- grouped-query attention over a sliding window with a logarithmic distance bias, query and
// key heads over their root mean squares, any head sizes.  Scores, weights and norms are fp32.
//
//   k_append    norms q and k of a prefill's rows, writes the key / value rows into the cache
//   k_wattn     plain form, any size and both activation types: one workgroup per (row, head), online softmax
//   k_wattn_m   bf16 MFMA form: 64 (position, head) pairs per workgroup against 64-key tiles of one key/value head
//   k_wattn_d   one new token per sequence: keys split over workgroups, partials merged by k_wattn_dc
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
// a wave per head of a row
template <typename T>
__global__ void __launch_bounds__(256) k_append(WAttnArgs a) {
    const int row = blockIdx.x, lane = threadIdx.x & 63;
    const int head = blockIdx.y * 4 + (threadIdx.x >> 6);
    if (head >= a.H + 2 * a.G) return;
    const SeqInfo q = a.seqs[a.row_seq[row]];
    const long pos = q.start + (row - q.off);
    const T* src = reinterpret_cast<const T*>(a.qkv) + (long)row * a.ldqkv;
    T* dst;
    int n, np;
    bool norm = true;
    if (head < a.H) {
        src += head * a.d; n = a.d; np = a.dp;
        dst = reinterpret_cast<T*>(a.q) + ((long)row * a.H + head) * a.dp;
    } else if (head < a.H + a.G) {
        const int g = head - a.H;
        src += a.H * a.d + g * a.d; n = a.d; np = a.dp;
        dst = reinterpret_cast<T*>(a.kc) + (((long)q.slot * a.G + g) * a.max_tokens + pos) * a.dp;
    } else {
        const int g = head - a.H - a.G;
        src += (a.H + a.G) * a.d + g * a.e; n = a.e; np = a.ep;
        dst = reinterpret_cast<T*>(a.vc) + (((long)q.slot * a.G + g) * a.max_tokens + pos) * a.ep;
        norm = false;
    }
    float inv = 1.0f;
    if (norm) {
        float ss = 0.0f;
        for (int i = lane; i < n; i += 64) {
            const float v = ldf(src + i);
            ss = fmaf(v, v, ss);
        }
        inv = 1.0f / sqrtf(wave_sum(ss) / (float)n + a.eps);
    }
    for (int i = lane; i < np; i += 64) stf(dst + i, i < n ? ldf(src + i) * inv : 0.0f);
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
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
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
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int j = j0 + t * 16 + 4 * lg + r;
                const int dist = i - j;
                const float s = biased(st[t][r], c1, r1, r2, (float)max(dist, 0));
                st[t][r] = (unsigned)dist < (unsigned)a.window ? s : -INFINITY;
                mt = fmaxf(mt, st[t][r]);
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
#pragma unroll
        for (int c = 0; c < DV / 16; ++c)
#pragma unroll
            for (int r = 0; r < 4; ++r) o[c][r] *= alpha;
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

// merge a head's partials: grid (H, B)
template <typename T>
__global__ void __launch_bounds__(256) k_wattn_dc(WAttnDecodeArgs a) {
    const int h = blockIdx.x, b = blockIdx.y, rs = a.ep + 2;
    const float* p = a.part + ((long)b * a.H + h) * a.nsplit * rs;
    float m = kNone;
    for (int s = 0; s < a.nsplit; ++s) m = fmaxf(m, p[(long)s * rs + a.ep]);
    float l = 0.0f;
    for (int s = 0; s < a.nsplit; ++s) l += p[(long)s * rs + a.ep + 1] * exp2f(p[(long)s * rs + a.ep] - m);
    T* o = reinterpret_cast<T*>(a.o) + (long)b * a.ldo;
    for (int c = threadIdx.x; c < a.e; c += 256) {
        float t = 0.0f;
        for (int s = 0; s < a.nsplit; ++s) {
            if (p[(long)s * rs + a.ep + 1] > 0.0f) t = fmaf(p[(long)s * rs + c], exp2f(p[(long)s * rs + a.ep] - m), t);
        }
        stf(o + h * a.e + c, t / l);
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
    const dim3 grid(a.rows, (a.H + 2 * a.G + 3) / 4);
    if (act == ACT_F32) hipLaunchKernelGGL((k_append<float>), grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((k_append<uint16_t>), grid, dim3(256), 0, s, a);
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
    const int tiles = (span + DK - 1) / DK;
    int n = (512 + B * G - 1) / (B * G);
    return std::max(1, std::min(std::min(n, tiles), 64));
}

size_t wattn_decode_floats(int B, int H, int ep, int nsplit) { return (size_t)B * H * nsplit * (ep + 2); }

void wattn_decode(hipStream_t s, Act act, const WAttnDecodeArgs& a) {
    if (act == ACT_F32) decode_t<float>(s, a);
    else decode_t<uint16_t>(s, a);
}

}  // namespace pgmi
