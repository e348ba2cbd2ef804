// Minimal JSON reader for model folders (config.json, the header of model.safetensors).  Host only.
#pragma once

#include <stdlib.h>
#include <string.h>

#include <string>
#include <utility>
#include <vector>

struct TgJson {
	enum Kind { Null, Bool, Number, String, Array, Object } kind = Null;
	bool b = false;
	double num = 0.0;
	std::string str;
	std::vector<TgJson> items;                            // Array
	std::vector<std::pair<std::string, TgJson>> members;  // Object

	const TgJson *get(const char *key) const {
		for (const auto &m : members)
			if (m.first == key) return &m.second;
		return nullptr;
	}
	bool is_object() const { return kind == Object; }
	bool is_null() const { return kind == Null; }

	// false: not JSON (err says where)
	static bool parse(const char *text, size_t n, TgJson *out, std::string *err) {
		Reader r{text, text + n, text};
		if (!r.value(out, 0)) {
			*err = "JSON error near byte " + std::to_string(r.p - text);
			return false;
		}
		r.space();
		if (r.p != r.end) {
			*err = "JSON: text behind the value at byte " + std::to_string(r.p - text);
			return false;
		}
		return true;
	}

private:
	struct Reader {
		const char *begin, *end, *p;
		void space() {
			while (p < end && (*p == ' ' || *p == '\n' || *p == '\t' || *p == '\r')) p++;
		}
		bool word(const char *w) {
			const size_t n = strlen(w);
			if ((size_t)(end - p) < n || memcmp(p, w, n) != 0) return false;
			p += n;
			return true;
		}
		static void utf8(std::string &s, unsigned c) {
			if (c < 0x80) s += (char)c;
			else if (c < 0x800) { s += (char)(0xC0 | (c >> 6)); s += (char)(0x80 | (c & 63)); }
			else { s += (char)(0xE0 | (c >> 12)); s += (char)(0x80 | ((c >> 6) & 63)); s += (char)(0x80 | (c & 63)); }
		}
		bool string(std::string *s) {
			if (p >= end || *p != '"') return false;
			for (p++; p < end && *p != '"'; p++) {
				if (*p != '\\') {
					*s += *p;
					continue;
				}
				if (++p >= end) return false;
				switch (*p) {
					case 'n': *s += '\n'; break;
					case 't': *s += '\t'; break;
					case 'r': *s += '\r'; break;
					case 'b': *s += '\b'; break;
					case 'f': *s += '\f'; break;
					case 'u': {
						if (end - p < 5) return false;
						const std::string hex(p + 1, 4);
						char *e = nullptr;
						utf8(*s, (unsigned)strtoul(hex.c_str(), &e, 16));
						if (*e) return false;
						p += 4;
						break;
					}
					default: *s += *p;
				}
			}
			if (p >= end) return false;
			p++;
			return true;
		}
		bool value(TgJson *v, int depth) {
			if (depth > 64) return false;
			space();
			if (p >= end) return false;
			if (*p == '{') {
				v->kind = Object;
				p++;
				space();
				if (p < end && *p == '}') { p++; return true; }
				for (;;) {
					space();
					std::pair<std::string, TgJson> m;
					if (!string(&m.first)) return false;
					space();
					if (p >= end || *p++ != ':') return false;
					if (!value(&m.second, depth + 1)) return false;
					v->members.push_back(std::move(m));
					space();
					if (p >= end) return false;
					if (*p == ',') { p++; continue; }
					return *p++ == '}';
				}
			}
			if (*p == '[') {
				v->kind = Array;
				p++;
				space();
				if (p < end && *p == ']') { p++; return true; }
				for (;;) {
					v->items.emplace_back();
					if (!value(&v->items.back(), depth + 1)) return false;
					space();
					if (p >= end) return false;
					if (*p == ',') { p++; continue; }
					return *p++ == ']';
				}
			}
			if (*p == '"') {
				v->kind = String;
				return string(&v->str);
			}
			if (word("true")) { v->kind = Bool; v->b = true; return true; }
			if (word("false")) { v->kind = Bool; return true; }
			if (word("null")) return true;
			const char *s = p;
			while (p < end && strchr("+-0123456789.eE", *p)) p++;
			if (p == s || p - s > 63) return false;
			const std::string t(s, p);
			char *e = nullptr;
			v->num = strtod(t.c_str(), &e);
			v->kind = Number;
			return *e == 0;
		}
	};
};
