// delta_rule.hip -- the gated delta rule over a ragged step: a matrix memory S per head that decays, is read at the token's key, corrected
// towards the token's value and read at the token's query.
//
// k_delta_prep  everything a token needs before the recurrence, in one launch: the causal short convolution + SiLU on q, k and v (the
//               carried tail moves on), unit vectors per query / key head, the product q . k, beta, the decay per head or key channel.  A wave per unit of work:
//               a query head with its key head (lanes over the coordinates), 256 value channels, 256 decays, the betas.
// k_delta_scan  a workgroup per (sequence, head, group of value columns).  Columns of S never meet, so every column walks the tokens on its
//               own: NGL neighbouring lanes hold a column, NPT numbers each, and meet in two DPP butterflies per token.  With a = g S the
//               token needs only the sums a.k and a.q at once:  u = beta (v - a.k),  S = a + k u,  o = a.q + (q.k) u.
//               The state lies (head, column, key coordinate), so a lane's numbers are 16-byte runs.
// All of it is fp32 in both serving formats.
#include "seq_common.h"

namespace {

constexpr int kMaxR = 8;             // coordinates of a query / key head per lane in k_delta_prep: dim <= 64 * kMaxR

struct PrepP {
    const float* proj; int64_t ld; int col0;                 // [q (kv_heads * dim) | k (kv_heads * dim) | v (heads * vdim)] of a projection row
    const float* w; float* tail; int taps;                   // (channels, taps); (slots, taps - 1, channels)
    int heads, kv_heads, dim, vdim;
    float q_scale, unit_eps;
    int b_col0;                                              // beta's columns of the same rows
    const float* z; int64_t ldz; int z_col0;                 // what the decay is computed from: heads numbers per token, or heads * dim
    const float* z_bias; const float* rate;                  // z_bias nullable, one per number of z; rate (heads): g = exp(-rate softplus(z + z_bias))
    int per_channel;
    float* qkv; float* qk; float* beta; float* decay;
};

__global__ __launch_bounds__(256) void k_delta_prep(const PrepP p, const zls_batch_t b) {
    const int t = blockIdx.x, lane = threadIdx.x & 63;
    const int sq = b.tok_seq[t];
    const int first = b.seq_start[sq], count = b.seq_start[sq + 1] - first;
    const int i0 = t - first, taps = p.taps;
    const int G = p.kv_heads, d = p.dim, V = p.heads * p.vdim, C = 2 * G * d + V, D = p.per_channel ? p.heads * d : p.heads;
    const int nv = (V + 255) / 256, nd = (D + 255) / 256, units = G + nv + nd + 1;
    float* tl = p.tail + (size_t)b.seq_slot[sq] * (taps - 1) * C;
    // the workgroups of a portion's first token also convolve its tokens up to taps - 2 -- the only ones that look into the tail -- and then
    // move the portion's last inputs into it (a lane owns its channels: rows in increasing order, each read before it is overwritten)
    const bool conv = i0 == 0 || i0 >= taps - 1;
    const int n = i0 == 0 ? max(1, min(count, taps - 1)) : 1;
    auto input = [&](int src, int c) {                       // src = -1 is the newest tail row
        return src >= 0 ? p.proj[(size_t)(first + src) * p.ld + p.col0 + c] : tl[(size_t)(taps - 1 + src) * C + c];
    };
    auto channel = [&](int i, int c) {
        float a = 0.f;
        for (int j = 0; j < taps; ++j) a = fmaf(p.w[(size_t)c * taps + j], input(i - (taps - 1 - j), c), a);
        return seq_silu(a);
    };
    auto shift = [&](int c) {
        for (int j = 0; j < taps - 1; ++j) tl[(size_t)j * C + c] = input(count - (taps - 1) + j, c);
    };
    for (int u = blockIdx.y * 4 + (threadIdx.x >> 6); u < units; u += gridDim.y * 4) {
        if (u < G) {
            if (!conv) continue;
            const int qc = u * d, kc = (G + u) * d;
            for (int i = i0; i < i0 + n; ++i) {
                float q[kMaxR], k[kMaxR], sq2 = 0.f, sk2 = 0.f, dot = 0.f;
#pragma unroll
                for (int r = 0; r < kMaxR; ++r) {
                    q[r] = k[r] = 0.f;
                    if (64 * r < d && lane + 64 * r < d) {
                        q[r] = channel(i, qc + lane + 64 * r);
                        k[r] = channel(i, kc + lane + 64 * r);
                    }
                    sq2 = fmaf(q[r], q[r], sq2);
                    sk2 = fmaf(k[r], k[r], sk2);
                    dot = fmaf(q[r], k[r], dot);
                }
                const float fq = p.q_scale / sqrtf(zl_wave_sum(sq2) + p.unit_eps), fk = 1.0f / sqrtf(zl_wave_sum(sk2) + p.unit_eps);
                dot = zl_wave_sum(dot) * fq * fk;
                float* row = p.qkv + (size_t)(first + i) * C;
#pragma unroll
                for (int r = 0; r < kMaxR; ++r)
                    if (64 * r < d && lane + 64 * r < d) {
                        row[qc + lane + 64 * r] = q[r] * fq;
                        row[kc + lane + 64 * r] = k[r] * fk;
                    }
                if (lane == 0) p.qk[(size_t)(first + i) * G + u] = dot;
            }
            if (i0 == 0)
                for (int e = lane; e < d; e += 64) { shift(qc + e); shift(kc + e); }
        } else if (u < G + nv) {
            if (!conv) continue;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int e = (u - G) * 256 + r * 64 + lane;
                if (e >= V) continue;
                const int c = 2 * G * d + e;
                for (int i = i0; i < i0 + n; ++i) p.qkv[(size_t)(first + i) * C + c] = channel(i, c);
                if (i0 == 0) shift(c);
            }
        } else if (u < G + nv + nd) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int e = (u - G - nv) * 256 + r * 64 + lane;
                if (e >= D) continue;
                const float z = p.z[(size_t)t * p.ldz + p.z_col0 + e] + (p.z_bias ? p.z_bias[e] : 0.f);
                p.decay[(size_t)t * D + e] = expf(-p.rate[p.per_channel ? e / d : e] * seq_softplus(z));
            }
        } else {
            for (int h = lane; h < p.heads; h += 64) p.beta[(size_t)t * p.heads + h] = seq_sigmoid(p.proj[(size_t)t * p.ld + p.b_col0 + h]);
        }
    }
}

struct DeltaP {
    const float* qkv; const float* qk; const float* beta; const float* decay;
    float* state; float* y;
    int heads, kv_heads, dim, vdim, chunk, vec;               // chunk: tokens staged at a time; vec: rows of q, k, decay and state in 16-byte pieces
};

constexpr int kSlotsKQ = 8, kSlotsG = 4, kSlotsS = 10;       // register slots of a thread for the next chunk: 16-byte pieces of q / k, of the decay, single numbers

template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
    return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
// the sum over NGL neighbouring lanes, in every lane: quads by permutation (xor 1, xor 2), then mirrored halves and rows of 16
template <int NGL>
__device__ __forceinline__ float group_sum(float v) {
    v = dpp_add<0xB1>(v);
    v = dpp_add<0x4E>(v);
    if constexpr (NGL >= 8) v = dpp_add<0x141>(v);
    if constexpr (NGL >= 16) v = dpp_add<0x140>(v);
    if constexpr (NGL >= 32) v += __shfl_xor(v, 16, 64);
    if constexpr (NGL >= 64) v += __shfl_xor(v, 32, 64);
    return v;
}

__device__ __forceinline__ float4 load4(const float* p, int n, int vec) {      // up to 4 numbers, n of them there
    if (vec) return *reinterpret_cast<const float4*>(p);
    return make_float4(p[0], n > 1 ? p[1] : 0.f, n > 2 ? p[2] : 0.f, n > 3 ? p[3] : 0.f);
}

// NGL lanes per column, NPT numbers per lane (coordinates 4 (g + NGL i) + e), CPL columns per group of lanes, PC: a decay per key channel.
// The tokens go through two LDS buffers of `chunk` rows [k | q | decay | v of the workgroup's columns | beta, decay, q.k]; the next chunk's
// loads are in flight while the current one is walked, and a token's row is read into registers one token ahead.
template <int NGL, int NPT, int CPL, bool PC>
__global__ __launch_bounds__(256) void k_delta_scan(const DeltaP p, const zls_batch_t b) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    constexpr int F = NPT / 4, DP = NGL * NPT, RUNS = PC ? 3 : 2;
    const int tid = threadIdx.x, nthr = blockDim.x, g = tid % NGL, ci = tid / NGL, groups = nthr / NGL;
    const int sq = blockIdx.x, h = blockIdx.y, hk = h / (p.heads / p.kv_heads), cols = groups * CPL, p0 = blockIdx.z * cols;
    const int d = p.dim, d4 = (d + 3) / 4, P = p.vdim, CH = p.chunk;
    const int first = b.seq_start[sq], count = b.seq_start[sq + 1] - first;
    const int WL = RUNS * DP + ((cols + 3) & ~3) + 4, VO = RUNS * DP, SO = WL - 4;
    const int qk_dim = p.kv_heads * d, C = 2 * qk_dim + p.heads * P;
    const int buf = (CH + 1) * WL;                           // (one row more: the walk reads a token ahead)
    for (int i = tid; i < 2 * buf; i += nthr) lds[i] = 0.f;

    // where a slot's numbers come from, relative to the chunk's first token, and where they go in a buffer; -1: nothing
    int ks[kSlotsKQ], kd[kSlotsKQ], gs[kSlotsG], gd[kSlotsG], ss[kSlotsS], sd[kSlotsS];
#pragma unroll
    for (int u = 0; u < kSlotsKQ; ++u) {
        const int e = tid + u * nthr, i = e / (2 * d4), r = e % (2 * d4), q = r / d4, f = r % d4;
        ks[u] = i < CH ? i * C + (q ? 0 : qk_dim) + hk * d + 4 * f : -1;
        kd[u] = i * WL + q * DP + 4 * f;
    }
    if constexpr (PC) {
#pragma unroll
        for (int u = 0; u < kSlotsG; ++u) {
            const int e = tid + u * nthr, i = e / d4, f = e % d4;
            gs[u] = i < CH ? (i * p.heads + h) * d + 4 * f : -1;
            gd[u] = i * WL + 2 * DP + 4 * f;
        }
    }
#pragma unroll
    for (int u = 0; u < kSlotsS; ++u) {
        const int e = tid + u * nthr, i = e / (cols + 3), c = e % (cols + 3);
        ss[u] = i < CH ? i : -1;
        sd[u] = c;
        if (i < CH && c < cols && p0 + c >= P) ss[u] = -1;   // (a column past the head's last: its zeros stay)
    }
    float4 kr[kSlotsKQ], gr[kSlotsG];
    float sr[kSlotsS];
    const int nk = (CH * 2 * d4 + nthr - 1) / nthr, ng = (CH * d4 + nthr - 1) / nthr, ns = (CH * (cols + 3) + nthr - 1) / nthr;
    auto fetch = [&](int c0) {
        const int cn = min(CH, count - c0);
        const float* base = p.qkv + (size_t)(first + c0) * C;
#pragma unroll
        for (int u = 0; u < kSlotsKQ; ++u)
            if (u < nk && ks[u] >= 0 && kd[u] < cn * WL) kr[u] = load4(base + ks[u], d - kd[u] % WL % DP, p.vec);
        if constexpr (PC) {
            const float* gb = p.decay + (size_t)(first + c0) * p.heads * d;
#pragma unroll
            for (int u = 0; u < kSlotsG; ++u)
                if (u < ng && gs[u] >= 0 && gd[u] < cn * WL) gr[u] = load4(gb + gs[u], d - (gd[u] % WL - 2 * DP), p.vec);
        }
#pragma unroll
        for (int u = 0; u < kSlotsS; ++u)
            if (u < ns && ss[u] >= 0 && ss[u] < cn) {
                const size_t tok = (size_t)(first + c0 + ss[u]);
                const int c = sd[u] - cols;
                if (c < 0) sr[u] = p.qkv[tok * C + 2 * qk_dim + h * P + p0 + sd[u]];
                else if (c == 0) sr[u] = p.beta[tok * p.heads + h];
                else if (c == 1) sr[u] = PC ? 1.0f : p.decay[tok * p.heads + h];
                else sr[u] = p.qk[tok * p.kv_heads + hk];
            }
    };
    auto publish = [&](int c0, float* dst) {
        const int cn = min(CH, count - c0);
#pragma unroll
        for (int u = 0; u < kSlotsKQ; ++u)
            if (u < nk && ks[u] >= 0 && kd[u] < cn * WL) *reinterpret_cast<float4*>(dst + kd[u]) = kr[u];
        if constexpr (PC) {
#pragma unroll
            for (int u = 0; u < kSlotsG; ++u)
                if (u < ng && gs[u] >= 0 && gd[u] < cn * WL) *reinterpret_cast<float4*>(dst + gd[u]) = gr[u];
        }
#pragma unroll
        for (int u = 0; u < kSlotsS; ++u)
            if (u < ns && ss[u] >= 0 && ss[u] < cn) dst[ss[u] * WL + (sd[u] < cols ? VO + sd[u] : SO + sd[u] - cols)] = sr[u];
    };

    fetch(0);
    float* st = p.state + ((size_t)b.seq_slot[sq] * p.heads + h) * P * d;
    float S[CPL][NPT];
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
        const int col = p0 + ci + c * groups;
#pragma unroll
        for (int i = 0; i < F; ++i) {
            const int n = 4 * (g + NGL * i);
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (col < P && n < d) v = load4(st + (size_t)col * d + n, d - n, p.vec);
            S[c][4 * i] = v.x; S[c][4 * i + 1] = v.y; S[c][4 * i + 2] = v.z; S[c][4 * i + 3] = v.w;
        }
    }
    __syncthreads();                                         // the buffers are zero
    publish(0, lds);
    __syncthreads();
    for (int c0 = 0, which = 0; c0 < count; c0 += CH, which ^= 1) {
        const int cn = min(CH, count - c0);
        const bool more = c0 + CH < count;
        if (more) fetch(c0 + CH);                            // in flight during the walk
        const float* rows = lds + which * buf;
        float4 kf[F], qf[F], gf[F], sc;
        float vv[CPL];
        auto read = [&](int i) {
            const float* row = rows + i * WL;
#pragma unroll
            for (int f = 0; f < F; ++f) {
                kf[f] = *reinterpret_cast<const float4*>(row + 4 * (g + NGL * f));
                qf[f] = *reinterpret_cast<const float4*>(row + DP + 4 * (g + NGL * f));
                if constexpr (PC) gf[f] = *reinterpret_cast<const float4*>(row + 2 * DP + 4 * (g + NGL * f));
            }
            sc = *reinterpret_cast<const float4*>(row + SO);
#pragma unroll
            for (int c = 0; c < CPL; ++c) vv[c] = row[VO + ci + c * groups];
        };
        read(0);
        for (int i = 0; i < cn; ++i) {
            float k[NPT], dk[CPL], dq[CPL], v[CPL];
            const float beta = sc.x, qk = sc.z;
#pragma unroll
            for (int c = 0; c < CPL; ++c) {
                float k0 = 0.f, k1 = 0.f, q0 = 0.f, q1 = 0.f;
#pragma unroll
                for (int f = 0; f < F; ++f) {
                    const float4 gg = PC ? gf[f] : make_float4(sc.y, sc.y, sc.y, sc.y);
                    float* s = S[c] + 4 * f;
                    s[0] *= gg.x; s[1] *= gg.y; s[2] *= gg.z; s[3] *= gg.w;
                    k0 = fmaf(s[0], kf[f].x, k0); k1 = fmaf(s[1], kf[f].y, k1); k0 = fmaf(s[2], kf[f].z, k0); k1 = fmaf(s[3], kf[f].w, k1);
                    q0 = fmaf(s[0], qf[f].x, q0); q1 = fmaf(s[1], qf[f].y, q1); q0 = fmaf(s[2], qf[f].z, q0); q1 = fmaf(s[3], qf[f].w, q1);
                }
                dk[c] = k0 + k1; dq[c] = q0 + q1; v[c] = vv[c];
            }
#pragma unroll
            for (int f = 0; f < F; ++f) { k[4 * f] = kf[f].x; k[4 * f + 1] = kf[f].y; k[4 * f + 2] = kf[f].z; k[4 * f + 3] = kf[f].w; }
            read(i + 1);
#pragma unroll
            for (int c = 0; c < CPL; ++c) { dk[c] = group_sum<NGL>(dk[c]); dq[c] = group_sum<NGL>(dq[c]); }
#pragma unroll
            for (int c = 0; c < CPL; ++c) {
                const float u = beta * (v[c] - dk[c]);
#pragma unroll
                for (int j = 0; j < NPT; ++j) S[c][j] = fmaf(k[j], u, S[c][j]);
                const int col = p0 + ci + c * groups;
                if (g == 0 && col < P) p.y[((size_t)(first + c0 + i) * p.heads + h) * P + col] = fmaf(qk, u, dq[c]);
            }
        }
        if (more) publish(c0 + CH, lds + (which ^ 1) * buf); // (the buffer of the chunk before: everybody passed the barrier behind its walk)
        __syncthreads();
    }
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
        const int col = p0 + ci + c * groups;
#pragma unroll
        for (int i = 0; i < F; ++i) {
            const int n = 4 * (g + NGL * i);
            if (col >= P || n >= d) continue;
            float* o = st + (size_t)col * d + n;
            if (p.vec) {
                *reinterpret_cast<float4*>(o) = make_float4(S[c][4 * i], S[c][4 * i + 1], S[c][4 * i + 2], S[c][4 * i + 3]);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (n + e < d) o[e] = S[c][4 * i + e];
            }
        }
    }
}

}  // namespace

extern "C" int zls_delta_prep(const float* proj, int64_t ld, int64_t col0, const float* w, float* tail, int64_t taps, int64_t heads, int64_t kv_heads,
                              int64_t dim, int64_t vdim, float q_scale, float unit_eps, int64_t b_col0, const float* z, int64_t ldz, int64_t z_col0,
                              const float* z_bias, const float* rate, int per_channel, const zls_batch_t* b, float* qkv, float* qk, float* beta,
                              float* decay, zl_stream_t s) {
    ZL_CHECK_ARG(proj && w && z && rate && qkv && qk && beta && decay && seq_batch_ok(b) && taps > 0 && (tail || taps == 1), ZL_EINVAL);
    ZL_CHECK_ARG(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0, ZL_ESHAPE);
    const int64_t C = 2 * kv_heads * dim + heads * vdim, D = per_channel ? heads * dim : heads;
    ZL_CHECK_ARG(col0 >= 0 && col0 + C <= ld && b_col0 >= 0 && b_col0 + heads <= ld && z_col0 >= 0 && z_col0 + D <= ldz, ZL_ESHAPE);
    ZL_CHECK_ARG(dim <= 64 * kMaxR && C < (1 << 28) && D < (1 << 28), ZL_ELIMIT);
    PrepP p = {};
    p.proj = proj; p.ld = ld; p.col0 = (int)col0; p.w = w; p.tail = tail; p.taps = (int)taps; p.heads = (int)heads; p.kv_heads = (int)kv_heads;
    p.dim = (int)dim; p.vdim = (int)vdim; p.q_scale = q_scale; p.unit_eps = unit_eps; p.b_col0 = (int)b_col0; p.z = z; p.ldz = ldz;
    p.z_col0 = (int)z_col0; p.z_bias = z_bias; p.rate = rate; p.per_channel = per_channel ? 1 : 0; p.qkv = qkv; p.qk = qk; p.beta = beta; p.decay = decay;
    const int64_t units = kv_heads + (heads * vdim + 255) / 256 + (D + 255) / 256 + 1, want = (units + 3) / 4;
    const int64_t most = b->n_tok > 512 ? 4 : 64;            // (a wave takes several units when the tokens alone fill the chip)
    hipLaunchKernelGGL(k_delta_prep, dim3(b->n_tok, (unsigned)(want < most ? want : most)), dim3(256), 0, (hipStream_t)s, p, *b);
    return zl_launch_status();
}

extern "C" int zls_delta_scan(const float* qkv, const float* qk, const float* beta, const float* decay, int per_channel, float* state, int64_t heads,
                              int64_t kv_heads, int64_t dim, int64_t vdim, const zls_batch_t* b, float* y, zl_stream_t s) {
    ZL_CHECK_ARG(qkv && qk && beta && decay && state && y && seq_batch_ok(b), ZL_EINVAL);
    ZL_CHECK_ARG(heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0, ZL_ESHAPE);
    const int64_t C = 2 * kv_heads * dim + heads * vdim;
    ZL_CHECK_ARG(dim <= 512 && vdim <= (1 << 20) && C * 16 < (1LL << 31) && heads * dim * 16 < (1LL << 31), ZL_ELIMIT);
    DeltaP p = {};
    p.qkv = qkv; p.qk = qk; p.beta = beta; p.decay = decay; p.state = state; p.y = y; p.heads = (int)heads; p.kv_heads = (int)kv_heads;
    p.dim = (int)dim; p.vdim = (int)vdim;
    auto al = [](const void* q) { return ((uintptr_t)q & 15) == 0; };
    p.vec = (dim % 4 == 0 && C % 4 == 0 && al(qkv) && al(state) && (!per_channel || al(decay))) ? 1 : 0;
    const int ngl = dim <= 16 ? 4 : dim <= 32 ? 8 : dim <= 128 ? 16 : dim <= 256 ? 32 : 64, npt = dim <= 64 ? 4 : 8;
    // two columns per group of lanes once single ones fill the chip's 1024 SIMDs; 1 .. 4 waves per workgroup, enough workgroups for every CU
    const int64_t waves = (int64_t)b->n_seq * heads * ((vdim * ngl + 63) / 64);
    const int cpl = waves > 1024 && vdim * ngl > 64 ? 2 : 1;
    const int64_t w = waves / cpl;
    int nthr = w >= 2048 ? 256 : w >= 512 ? 128 : 64;
    while (nthr > 64 && (nthr / 2 / ngl) * cpl >= vdim) nthr /= 2;
    const int cols = nthr / ngl * cpl, d4 = (int)((dim + 3) / 4), runs = per_channel ? 3 : 2;
    int ch = 16;
    auto least = [&](int v) { if (v < ch) ch = v; };
    least(kSlotsKQ * nthr / (2 * d4));
    least(kSlotsG * nthr / d4);
    least(kSlotsS * nthr / (cols + 3));
    if (ch > b->max_count) ch = b->max_count;
    const size_t row = (size_t)(runs * ngl * npt + ((cols + 3) & ~3) + 4) * sizeof(float);
    while (ch > 1 && 2 * (ch + 1) * row > 64 * 1024) --ch;
    ZL_CHECK_ARG(ch >= 1, ZL_ELIMIT);
    p.chunk = ch;
    const size_t lds = 2 * (ch + 1) * row;
    ZL_CHECK_ARG(lds <= 64 * 1024, ZL_ELIMIT);
    const int64_t parts = (vdim + cols - 1) / cols;
    ZL_CHECK_ARG(parts <= 65535, ZL_ELIMIT);
    const dim3 grid((unsigned)b->n_seq, (unsigned)heads, (unsigned)parts);
    hipStream_t hs = (hipStream_t)s;
#define GO(NGL, NPT, CPL, PC) hipLaunchKernelGGL((k_delta_scan<NGL, NPT, CPL, PC>), grid, dim3(nthr), lds, hs, p, *b)
#define SIZES(NGL, NPT)                                                                       \
    if (cpl == 2) { if (per_channel) GO(NGL, NPT, 2, true); else GO(NGL, NPT, 2, false); }    \
    else { if (per_channel) GO(NGL, NPT, 1, true); else GO(NGL, NPT, 1, false); }
    if (dim <= 16) { SIZES(4, 4) }
    else if (dim <= 32) { SIZES(8, 4) }
    else if (dim <= 64) { SIZES(16, 4) }
    else if (dim <= 128) { SIZES(16, 8) }
    else if (dim <= 256) { SIZES(32, 8) }
    else { SIZES(64, 8) }
#undef SIZES
#undef GO
    return zl_launch_status();
}
